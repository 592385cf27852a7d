// lm_latent.hip - kernels of the layer-list language models (see lm_latent.h): float32 residual stream, layer-scaled parallel branches,
// latent attention with a sliding window, rotary tables with YaRN scaling, and the true-float32 GEMM of the 32-bit mode.
//
// Latent attention.  A token leaves ONE cache row [c | k_r]: the RMS-normed latent c (R values, shared by all heads) and the rotated key
// part k_r (r values, shared by all heads).  Two algebraically equal forms are used:
//   absorbed (decode)   q_lat = W_uk^T q_plain;  score = q_lat . c + q_rot . k_r;  o_lat = sum_j p_j c_j;  out = W_uv o_lat
//                       - a decode step reads R + r values per cached token whatever the number of heads;
//   expanded (prompts)  k = W_uk c, v = W_uv c for every key row by one GEMM, then ordinary tiled attention with n + r and v dimensions
//                       - (n + r + v) instead of (2 R + r) multiplications per (query, key, head).
// Scores, the softmax and its weights are float32 in both; the weights enter the matrix cores as bf16 hi + lo pairs.
#include "lm_latent.h"
#include "lm_device.h"
#include <math.h>

// ============================================================================ rotary tables (host)
// Pair i of a rotated vector turns by pos * f_i, f_i = base^(-2 i / dims).  YaRN: a pair that turns more than `fast` times over the original
// context keeps f_i, one that turns less than `slow` times gets f_i / factor, a linear ramp over the pair index between; both cos and sin
// are multiplied by 0.1 ln(factor) + 1.
void rotary_tables_host(const RotarySpec& r, int positions, std::vector<float>& cos_out, std::vector<float>& sin_out) {
    const int half = r.dims / 2;
    std::vector<double> f(half);
    double mag = 1.0;
    for (int i = 0; i < half; ++i) f[i] = pow(r.base, -2.0 * i / r.dims);
    if (r.yarn) {
        auto dim_of_turns = [&](double turns) { return r.dims * log(r.original / (2.0 * M_PI * turns)) / (2.0 * log(r.base)); };
        const double lo = std::max(floor(dim_of_turns(r.fast)), 0.0), hi = std::min(ceil(dim_of_turns(r.slow)), (double)(r.dims - 1));
        for (int i = 0; i < half; ++i) {
            const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
            f[i] = f[i] / r.factor * ramp + f[i] * (1.0 - ramp);
        }
        mag = 0.1 * log(r.factor) + 1.0;
    }
    cos_out.resize((size_t)positions * half);
    sin_out.resize((size_t)positions * half);
    for (int p = 0; p < positions; ++p)
        for (int i = 0; i < half; ++i) {
            const double a = (double)p * f[i];
            cos_out[(size_t)p * half + i] = (float)(cos(a) * mag);
            sin_out[(size_t)p * half + i] = (float)(sin(a) * mag);
        }
}

extern "C" mis_status mis_debug_rotary_tables(int dims, double base, int yarn, double factor, double original, double fast, double slow, int positions,
                                              float* cos_out, float* sin_out) {
    MIS_API_BEGIN
    MIS_REQUIRE(dims >= 2 && dims % 2 == 0 && positions >= 1 && cos_out && sin_out, MIS_ERR_INVALID_INPUT, "bad argument");
    RotarySpec r{dims, base, yarn != 0, factor, original, fast, slow};
    std::vector<float> c, s;
    rotary_tables_host(r, positions, c, s);
    std::copy(c.begin(), c.end(), cos_out);
    std::copy(s.begin(), s.end(), sin_out);
    MIS_API_END
}

LatentDims latent_dims(int H, int n, int r, int v, int R, int window, int rot_dims, float scale, float eps) {
    LatentDims D{};
    D.H = H; D.n = n; D.r = r; D.v = v; D.R = R;
    D.np = (int)round_up(n, 32); D.rp = (int)round_up(r, 16); D.vp = (int)round_up(v, 16);
    D.Rp = std::max(128, (int)round_up(R, 64));
    D.CW = (int)round_up(D.Rp + D.rp, 32);
    D.DK = (int)round_up(D.np + D.rp, 32);
    D.window = window; D.rot_dims = rot_dims; D.scale = scale; D.eps = eps;
    return D;
}

// ============================================================================ embedding, residual + layer scale + norm
// CPT groups of four columns per thread; columns of the width padding (d .. dp) hold zeros everywhere (weights, tables, stream)
template <int CPT>
__global__ void __launch_bounds__(1024) k_rows_embed_norm2(const bf16_t* __restrict__ emb, const int32_t* __restrict__ ids, int vocab,
                                                           const bf16_t* __restrict__ g_embed, const bf16_t* __restrict__ g_norm, float* __restrict__ x,
                                                           Operand h, int d, int dp, float eps, float g_add, int n_rows, const uint8_t* __restrict__ on,
                                                           int32_t* __restrict__ pos_cur, int32_t* __restrict__ pos_next) {
    __shared__ float red[16];
    const int m = blockIdx.x, tid = threadIdx.x, nth = blockDim.x, nc = dp >> 2;
    int id = m < n_rows ? ids[m] : 0;
    if (id < 0 || id >= vocab) id = 0;
    if (pos_next && tid == 0 && m < n_rows) {
        const int p = pos_next[m];
        pos_cur[m] = p;
        if (on[m]) pos_next[m] = p + 1;
    }
    float e[CPT][4], ge[CPT][4], gn[CPT][4], ss = 0.0f;
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        const int c = tid + g * nth, cc = c < nc ? c : 0;
        load4_bf16(emb + (size_t)id * dp + 4 * cc, e[g]);
        load4_bf16((g_embed ? g_embed : g_norm) + 4 * cc, ge[g]);
        load4_bf16(g_norm + 4 * cc, gn[g]);
#pragma unroll
        for (int j = 0; j < 4; ++j) ss += c < nc ? e[g][j] * e[g][j] : 0.0f;
    }
    const float inv = 1.0f / sqrtf(lat_block_sum(ss, red) / (float)d + eps);
    float s2 = 0.0f;
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        const int c = tid + g * nth;
#pragma unroll
        for (int j = 0; j < 4; ++j) { if (g_embed) e[g][j] = e[g][j] * inv * ge[g][j]; s2 += c < nc ? e[g][j] * e[g][j] : 0.0f; }
        if (c < nc) *reinterpret_cast<float4*>(x + (size_t)m * dp + 4 * c) = make_float4(e[g][0], e[g][1], e[g][2], e[g][3]);
    }
    const float inv2 = 1.0f / sqrtf(lat_block_sum(s2, red) / (float)d + eps);
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        const int c = tid + g * nth;
        float o[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) o[j] = e[g][j] * inv2 * (gn[g][j] + g_add);
        if (c < nc) operand_store4(h, m, 4 * c, o);
    }
}

// SG >= s1 + s2 (clamped, unconditional loads: one round trip for everything the row needs); SG = 0: no slabs, the stream is only normed
template <int CPT, int SG>
__global__ void __launch_bounds__(1024) k_scaled_residual_norm(ScaledSlabs A, int slab_rows, float* __restrict__ x, const int32_t* __restrict__ row_of,
                                                               const bf16_t* __restrict__ g_norm, Operand h, int d, int dp, float eps, float g_add) {
    __shared__ float red[16];
    const int m = blockIdx.x, tid = threadIdx.x, nth = blockDim.x, nc = dp >> 2;
    const size_t xr = (size_t)(row_of ? row_of[m] : m) * dp;
    float v[CPT][4], gn[CPT][4], ss = 0.0f;
    float4 sl[CPT][SG ? SG : 1];
    float l1[CPT][4], l2[CPT][4];
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        const int c = tid + g * nth, cc = c < nc ? c : 0;
        const float4 t = *reinterpret_cast<const float4*>(x + xr + 4 * cc);
        v[g][0] = t.x; v[g][1] = t.y; v[g][2] = t.z; v[g][3] = t.w;
        load4_bf16(g_norm + 4 * cc, gn[g]);
        if constexpr (SG > 0) {
            const int S = A.s1 + A.s2;
#pragma unroll
            for (int j = 0; j < SG; ++j) sl[g][j] = *reinterpret_cast<const float4*>(A.p + ((size_t)(j < S ? j : S - 1) * slab_rows + m) * dp + 4 * cc);
            load4_bf16(A.ls1 + 4 * cc, l1[g]);
            load4_bf16((A.s2 ? A.ls2 : A.ls1) + 4 * cc, l2[g]);
        }
    }
    if constexpr (SG > 0) {
#pragma unroll
        for (int g = 0; g < CPT; ++g) {
            float a[4] = {0.f, 0.f, 0.f, 0.f}, b[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int j = 0; j < SG; ++j) {                       // slab order 0, 1, 2, ...: deterministic
                const bool first = j < A.s1, second = !first && j < A.s1 + A.s2;
                const float f[4] = {sl[g][j].x, sl[g][j].y, sl[g][j].z, sl[g][j].w};
#pragma unroll
                for (int e = 0; e < 4; ++e) { a[e] += first ? f[e] : 0.0f; b[e] += second ? f[e] : 0.0f; }
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) v[g][e] += l1[g][e] * a[e] + l2[g][e] * b[e];
            const int c = tid + g * nth;
            if (c < nc) *reinterpret_cast<float4*>(x + xr + 4 * c) = make_float4(v[g][0], v[g][1], v[g][2], v[g][3]);
        }
    }
#pragma unroll
    for (int g = 0; g < CPT; ++g)
#pragma unroll
        for (int j = 0; j < 4; ++j) ss += tid + g * nth < nc ? v[g][j] * v[g][j] : 0.0f;
    const float inv = 1.0f / sqrtf(lat_block_sum(ss, red) / (float)d + eps);
#pragma unroll
    for (int g = 0; g < CPT; ++g) {
        const int c = tid + g * nth;
        float o[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) o[j] = v[g][j] * inv * (gn[g][j] + g_add);
        if (c < nc) operand_store4(h, m, 4 * c, o);
    }
}

int row_cpt(int dp) { const int nc = dp / 4; return nc <= 1024 ? (nc >= 512 ? 2 : 1) : (nc <= 2048 ? 2 : 4); }
int row_threads(int dp, int cpt) { return (int)round_up(cdiv(dp / 4, cpt), 64); }
void row_check(int dp) { MIS_REQUIRE(dp % 4 == 0 && dp <= 16384, MIS_ERR_INVALID_INPUT, "model width above 16384"); }

void launch_rows_embed_norm2(const bf16_t* emb, const int32_t* ids, int vocab, const bf16_t* g_embed, const bf16_t* g_norm, float* x, const Operand& h,
                             int d, int dp, float eps, int n_rows, int rows, const uint8_t* on, int32_t* pos_cur, int32_t* pos_next, hipStream_t s, float g_add) {
    row_check(dp);
    const int cpt = row_cpt(dp), nth = row_threads(dp, cpt);
#define EMB2(C) hipLaunchKernelGGL((k_rows_embed_norm2<C>), dim3(rows), dim3(nth), 0, s, emb, ids, vocab, g_embed, g_norm, x, h, d, dp, eps, g_add, n_rows, on, pos_cur, pos_next)
    if (cpt == 1) EMB2(1); else if (cpt == 2) EMB2(2); else EMB2(4);
#undef EMB2
}
static void residual_norm(const ScaledSlabs& a, int slab_rows, float* x, const int32_t* row_of, const bf16_t* g_norm, const Operand& h, int d, int dp,
                          float eps, float g_add, int rows, hipStream_t s) {
    row_check(dp);
    const int cpt = row_cpt(dp), nth = row_threads(dp, cpt), S = a.s1 + a.s2;
    MIS_REQUIRE(S <= (cpt == 4 ? 4 : 8), MIS_ERR_GENERATION_FAILED, "too many split-K slabs");
#define RN(C, G) hipLaunchKernelGGL((k_scaled_residual_norm<C, G>), dim3(rows), dim3(nth), 0, s, a, slab_rows, x, row_of, g_norm, h, d, dp, eps, g_add)
#define RNC(C) do { if (S == 0) RN(C, 0); else if (S <= 2) RN(C, 2); else if (S <= 4) RN(C, 4); else RN(C, C == 4 ? 4 : 8); } while (0)
    if (cpt == 1) RNC(1); else if (cpt == 2) RNC(2); else RNC(4);
#undef RNC
#undef RN
}
void launch_scaled_residual_norm(const ScaledSlabs& a, int slab_rows, float* x, const bf16_t* g_norm, const Operand& h, int d, int dp, float eps, int rows,
                                 hipStream_t s) {
    residual_norm(a, slab_rows, x, nullptr, g_norm, h, d, dp, eps, 0.0f, rows, s);
}
void launch_gather_norm(const float* x, const int32_t* row_of, const bf16_t* g_norm, const Operand& h, int d, int dp, float eps, int rows, hipStream_t s, float g_add) {
    residual_norm(ScaledSlabs{}, 0, const_cast<float*>(x), row_of, g_norm, h, d, dp, eps, g_add, rows, s);
}

// ============================================================================ float32 GEMM (v_mfma_f32_16x16x4_f32)
// Weight tiles are the bf16 fragments of the other GEMMs: lane q*16 + i holds W[16 nt + i][32 kt + 8 q .. + 8].  Taking element e of every lane
// as one K = 4 step (k = 8 q + e for q = 0..3) needs no re-layout; the other operand is read as X[m][32 kt + 8 q + e].
template <int EPI>
__global__ void __launch_bounds__(256) k_gemm_f32(GemmF32 g) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int nt = blockIdx.x * 4 + wave, m0 = blockIdx.y * 64, z = blockIdx.z;
    if (nt >= g.NT) return;
    const int li = lane & 15, q = lane >> 4;
    const bf16_t* wp = g.W + g.wz * z + ((size_t)nt * g.KT * 64 + lane) * 8;
    const float* xp[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) xp[j] = g.X + g.xz * z + (size_t)min(m0 + j * 16 + li, g.M - 1) * g.ldx + q * 8;
    f32x4_t acc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[j] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    for (int kt = 0; kt < g.KT; ++kt) {
        const bf16x8_t w = *reinterpret_cast<const bf16x8_t*>(wp + (size_t)kt * 512);
        float wf[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) wf[e] = bf16_to_f32((bf16_t)w[e]);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const float4 a = *reinterpret_cast<const float4*>(xp[j] + kt * 32), b = *reinterpret_cast<const float4*>(xp[j] + kt * 32 + 4);
            const float xf[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(wf[e], xf[e], acc[j], 0, 0, 0);
        }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int m = m0 + j * 16 + li;
        if (m >= g.M) continue;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int n = nt * 16 + q * 4 + e;
            if (n >= g.n_valid) continue;
            float* o = g.out + (size_t)m * g.ldo + g.oz * z + n;
            const float v = acc[j][e];
            if (EPI == F32_STORE) *o = v;
            else if (EPI == F32_RELU2) { const float t = fmaxf(v, 0.0f); *o = t * t; }
            else if (EPI == F32_ADD_SCALED) *o += bf16_to_f32(g.ls[n]) * v;
            else { const float t = v * g.scale; *o = g.cap > 0.0f ? g.cap * tanhf(t / g.cap) : t; }
        }
    }
}
void launch_gemm_f32(const GemmF32& g, hipStream_t s) {
    MIS_REQUIRE(g.M >= 1 && g.NT >= 1 && g.KT >= 1 && g.ldx % 4 == 0 && g.xz % 4 == 0, MIS_ERR_GENERATION_FAILED, "float32 GEMM: bad shape");
    dim3 grid(cdiv(g.NT, 4), cdiv(g.M, 64), g.heads);
    if (g.epi == F32_STORE) hipLaunchKernelGGL((k_gemm_f32<F32_STORE>), grid, dim3(256), 0, s, g);
    else if (g.epi == F32_RELU2) hipLaunchKernelGGL((k_gemm_f32<F32_RELU2>), grid, dim3(256), 0, s, g);
    else if (g.epi == F32_ADD_SCALED) hipLaunchKernelGGL((k_gemm_f32<F32_ADD_SCALED>), grid, dim3(256), 0, s, g);
    else hipLaunchKernelGGL((k_gemm_f32<F32_SOFTCAP>), grid, dim3(256), 0, s, g);
}

// ============================================================================ projections -> cache row and query rows
// columns j .. j + 3 (j % 4 == 0) of a rotary part: pairs (2 i, 2 i + 1) below rot_dims are turned, the others pass (padding columns hold zeros)
__device__ __forceinline__ void rotary4(const float* src, int j, int rot_dims, const float* cs, const float* sn, float (&o)[4]) {
    const float4 t = *reinterpret_cast<const float4*>(src + j);
    o[0] = t.x; o[1] = t.y; o[2] = t.z; o[3] = t.w;
#pragma unroll
    for (int k = 0; k < 2; ++k)
        if (j + 2 * k < rot_dims) {
            const float c = cs[(j >> 1) + k], s = sn[(j >> 1) + k], u = o[2 * k], v = o[2 * k + 1];
            o[2 * k] = u * c - v * s;
            o[2 * k + 1] = v * c + u * s;
        }
}

template <typename T>
__device__ __forceinline__ void latent_row(const LatentDims& D, const LatentRows& p, int m, float* red) {
    const int tid = threadIdx.x, nth = blockDim.x, HQ = D.np + D.rp;
    if (p.rows.on && !p.rows.on[m]) return;                                    // block-uniform
    const int pos = p.rows.pos[m], seq = p.rows.seq ? p.rows.seq[m] : m;
    const float* row = p.qkv + (size_t)m * p.ld;
    const float* craw = row + (size_t)D.H * HQ;                                 // [latent Rp | rotary key rp], padding columns zero
    const float *cs = p.rope_cos + (size_t)pos * (D.rot_dims / 2), *sn = p.rope_sin + (size_t)pos * (D.rot_dims / 2);
    float ss = 0.0f;
    for (int i = tid * 4; i < D.Rp; i += nth * 4) {
        const float4 t = *reinterpret_cast<const float4*>(craw + i);
        ss += t.x * t.x + t.y * t.y + t.z * t.z + t.w * t.w;
    }
    // query rows (independent of the latent's norm)
    T* q = (T*)p.q + (size_t)m * D.H * p.q_ld;
    const int j0 = p.with_plain ? 0 : p.q_rot_off, w = (p.q_ld - j0) >> 2;
    for (int t = tid; t < D.H * w; t += nth) {
        const int hd = t / w, j = j0 + (t - hd * w) * 4, jr = j - p.q_rot_off;
        const float* src = row + (size_t)hd * HQ;
        float o[4] = {0.f, 0.f, 0.f, 0.f};
        if (jr < 0) { const float4 f = *reinterpret_cast<const float4*>(src + j); o[0] = f.x; o[1] = f.y; o[2] = f.z; o[3] = f.w; }
        else if (jr < D.rp) rotary4(src + D.np, jr, D.rot_dims, cs, sn, o);
        put4(q + (size_t)hd * p.q_ld + j, o);
    }
    const float inv = 1.0f / sqrtf(lat_block_sum(ss, red) / (float)D.R + D.eps);
    T* cache = (T*)p.cache + ((size_t)seq * p.Smax + pos) * D.CW;
    for (int i = tid * 4; i < D.CW; i += nth * 4) {
        float o[4] = {0.f, 0.f, 0.f, 0.f};
        if (i < D.Rp) {
            const float4 t = *reinterpret_cast<const float4*>(craw + i);
            float g[4];
            load4_bf16(p.c_norm + i, g);
            o[0] = t.x * inv * g[0]; o[1] = t.y * inv * g[1]; o[2] = t.z * inv * g[2]; o[3] = t.w * inv * g[3];
        } else if (i < D.Rp + D.rp) rotary4(craw + D.Rp, i - D.Rp, D.rot_dims, cs, sn, o);
        put4(cache + i, o);
    }
}
template <typename T>
__global__ void __launch_bounds__(256) k_latent_rows(LatentDims D, LatentRows p) {
    __shared__ float red[4];
    latent_row<T>(D, p, blockIdx.x, red);
}
static void latent_rows_check(const LatentDims& D, const LatentRows& p) {
    MIS_REQUIRE(p.rows.pos && p.Smax >= 1 && D.rot_dims % 2 == 0 && D.rot_dims <= D.r && p.q_rot_off + D.r <= p.q_ld && (!p.with_plain || p.q_rot_off == D.np),
                MIS_ERR_GENERATION_FAILED, "latent rows: bad layout");
}
void launch_latent_rows(const LatentDims& D, const LatentRows& p, int rows, hipStream_t s) {
    latent_rows_check(D, p);
    if (p.f32) hipLaunchKernelGGL((k_latent_rows<float>), dim3(rows), dim3(256), 0, s, D, p);
    else hipLaunchKernelGGL((k_latent_rows<bf16_t>), dim3(rows), dim3(256), 0, s, D, p);
}

// ---- per-head GEMM of a few rows: A = packed weight tiles of the head, B = rows (converted to bf16 fragments on the fly)
__device__ __forceinline__ bf16x8_t frag8(const float* p) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    const float f[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
    bf16x8_t r;
#pragma unroll
    for (int e = 0; e < 8; ++e) r[e] = (short)f32_to_bf16(f[e]);
    return r;
}
__device__ __forceinline__ bf16x8_t frag8(const bf16_t* p) { return *reinterpret_cast<const bf16x8_t*>(p); }

// two row tiles (32 rows from m0) x one weight tile over KT k-tiles, four k-tiles requested at a time
template <typename T>
__device__ __forceinline__ void head_tile(const T* X, size_t ldx, int m0, int rows, const bf16_t* wt, int KT, f32x4_t (&acc)[2]) {
    const int lane = threadIdx.x & 63, li = lane & 15, q = lane >> 4;
    const T* x0 = X + (size_t)min(m0 + li, rows - 1) * ldx + q * 8;
    const T* x1 = X + (size_t)min(m0 + 16 + li, rows - 1) * ldx + q * 8;
    acc[0] = acc[1] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < KT; k0 += 4) {
        bf16x8_t a[4], b0[4], b1[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int kt = min(k0 + u, KT - 1);
            a[u] = *reinterpret_cast<const bf16x8_t*>(wt + ((size_t)kt * 64 + lane) * 8);
            b0[u] = frag8(x0 + kt * 32); b1[u] = frag8(x1 + kt * 32);
        }
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            if (k0 + u >= KT) continue;
            acc[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u], b0[u], acc[0], 0, 0, 0);
            acc[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a[u], b1[u], acc[1], 0, 0, 0);
        }
    }
}

// blocks [0, n_abs): q_lat tiles (4 waves = 4 latent tiles of one head, 32 rows); blocks behind: one row each (latent_row)
__global__ void __launch_bounds__(256) k_latent_absorb(LatentDims D, LatentRows p, const bf16_t* __restrict__ uk_t, int rows, int n_abs, int mblocks) {
    __shared__ float red[4];
    if ((int)blockIdx.x >= n_abs) { latent_row<bf16_t>(D, p, blockIdx.x - n_abs, red); return; }
    const int tb = D.Rp / 64;                                                   // blocks of four latent tiles per head
    const int mb = blockIdx.x % mblocks, t = blockIdx.x / mblocks;
    const int hd = t / tb, rt = (t - hd * tb) * 4 + (threadIdx.x >> 6);
    const int KT = D.np / 32, HQ = D.np + D.rp, m0 = mb * 32;
    f32x4_t acc[2];
    head_tile<float>(p.qkv + (size_t)hd * HQ, p.ld, m0, rows, uk_t + ((size_t)hd * (D.Rp / 16) + rt) * KT * 512, KT, acc);
    const int lane = threadIdx.x & 63;
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int m = m0 + j * 16 + (lane & 15);
        if (m >= rows) continue;
        const float v[4] = {acc[j][0], acc[j][1], acc[j][2], acc[j][3]};
        *reinterpret_cast<uint2*>((bf16_t*)p.q + ((size_t)m * D.H + hd) * p.q_ld + rt * 16 + (lane >> 4) * 4) = pack4_bf16(v);
    }
}
void launch_latent_absorb(const LatentDims& D, const LatentRows& p, const bf16_t* uk_t, int rows, hipStream_t s) {
    latent_rows_check(D, p);
    MIS_REQUIRE(!p.f32 && !p.with_plain && p.q_rot_off == D.Rp && p.q_ld == D.CW && p.ld % 4 == 0, MIS_ERR_GENERATION_FAILED, "latent absorb: bad layout");
    const int mblocks = cdiv(rows, 32), n_abs = D.H * (D.Rp / 64) * mblocks;
    hipLaunchKernelGGL(k_latent_absorb, dim3(n_abs + rows), dim3(256), 0, s, D, p, uk_t, rows, n_abs, mblocks);
}

// one wave per (head, value tile, 32 rows)
__global__ void __launch_bounds__(256) k_latent_values(LatentDims D, const bf16_t* __restrict__ o_lat, const bf16_t* __restrict__ uv, size_t uvz, Operand out, int rows) {
    const int vt = D.vp / 16, item = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (item >= D.H * vt) return;
    const int hd = item / vt, t = item - hd * vt, m0 = blockIdx.y * 32, lane = threadIdx.x & 63, KT = D.Rp / 32;
    f32x4_t acc[2];
    head_tile<bf16_t>(o_lat + (size_t)hd * D.Rp, (size_t)D.H * D.Rp, m0, rows, uv + uvz * hd + (size_t)t * KT * 512, KT, acc);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int m = m0 + j * 16 + (lane & 15), c = t * 16 + (lane >> 4) * 4;
        if (m >= rows) continue;
        if (D.v % 4 == 0) {
            const float v[4] = {acc[j][0], acc[j][1], acc[j][2], acc[j][3]};
            if (c < D.v) operand_store4(out, m, hd * D.v + c, v);
        } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) if (c + e < D.v) operand_store1(out, m, hd * D.v + c + e, acc[j][e]);
        }
    }
}
void launch_latent_values(const LatentDims& D, const bf16_t* o_lat, const bf16_t* uv, size_t uvz, const Operand& out, int rows, hipStream_t s) {
    hipLaunchKernelGGL(k_latent_values, dim3(cdiv((int64_t)D.H * (D.vp / 16), 4), cdiv(rows, 32)), dim3(256), 0, s, D, o_lat, uv, uvz, out, rows);
}

// ============================================================================ absorbed attention, any sizes (float32 mode; bf16 sizes past the MFMA kernel)
#define LAT_OC 8                                   // latent columns per thread: Rp <= 256 * LAT_OC
template <typename T>
__global__ void __launch_bounds__(256) k_latent_attn_any(LatentDims D, LatentAttn p) {
    extern __shared__ float sm[];                  // q [CW] | weights [256] | red [8]
    float *sq = sm, *sw = sm + D.CW, *red = sw + 256;
    const int m = blockIdx.x, hd = blockIdx.y, tid = threadIdx.x, lane = tid & 63;
    T* out = (T*)p.out + ((size_t)m * D.H + hd) * D.Rp;
    if (p.rows.on && !p.rows.on[m]) { for (int i = tid; i < D.Rp; i += 256) put(out + i, 0.0f); return; }
    const int pos = p.rows.pos[m], seq = p.rows.seq ? p.rows.seq[m] : m;
    const int lo = D.window > 0 ? max(0, pos - D.window + 1) : 0;
    const T* q = (const T*)p.q + ((size_t)m * D.H + hd) * D.CW;
    const T* cache = (const T*)p.cache + (size_t)seq * p.Smax * D.CW;
    for (int i = tid; i < D.CW; i += 256) sq[i] = get(q + i);
    __syncthreads();
    float mx = -INFINITY, sum = 0.0f, acc[LAT_OC];
#pragma unroll
    for (int j = 0; j < LAT_OC; ++j) acc[j] = 0.0f;
    for (int k0 = lo; k0 <= pos; k0 += 256) {
        const int key = k0 + tid;
        float sc = -INFINITY;
        if (key <= pos) {
            const T* kr = cache + (size_t)key * D.CW;
            float a = 0.0f;
            for (int i = 0; i < D.CW; i += 8) {
#pragma unroll
                for (int e = 0; e < 8; ++e) a += sq[i + e] * get(kr + i + e);
            }
            sc = a * D.scale;
        }
        float cm = wave_max(sc);
        if (lane == 0) red[tid >> 6] = cm;
        __syncthreads();
        cm = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
        const float mn = fmaxf(mx, cm), alpha = expf(mx - mn);
        const float w = key <= pos ? expf(sc - mn) : 0.0f;
        sw[tid] = w;
        const float ws = wave_sum(w);
        if (lane == 0) red[4 + (tid >> 6)] = ws;
        __syncthreads();
        sum = sum * alpha + ((red[4] + red[5]) + (red[6] + red[7]));
        mx = mn;
        const int nk = min(256, pos - k0 + 1);
#pragma unroll
        for (int j = 0; j < LAT_OC; ++j) {
            const int c = tid + 256 * j;
            if (c >= D.Rp) continue;
            float a = acc[j] * alpha;
            for (int k = 0; k < nk; ++k) a += sw[k] * get(cache + (size_t)(k0 + k) * D.CW + c);
            acc[j] = a;
        }
        __syncthreads();
    }
#pragma unroll
    for (int j = 0; j < LAT_OC; ++j) {
        const int c = tid + 256 * j;
        if (c < D.Rp) put(out + c, acc[j] / sum);
    }
}

// ============================================================================ absorbed attention on the matrix cores (decode)
// Block = one row, HT tiles of 16 heads (four waves each), one share of the row's keys, walked in tiles of 64.  A key is read ONCE: each thread
// fetches 4 keys (kg, kg + 16, kg + 32, kg + 48) x 8 columns, writes them to LDS as key rows (score operand) and, transposed in registers, as
// column rows (value operand; key kg + 16 k at place 4 kg + k); the next tile's loads are in flight during the rest (barriers wait for LDS
// only).  The queries come through LDS too: a wave needs a head tile's whole query, four times what the block has to fetch.  Wave w of a head tile scores keys 16 w .. + 15
// (S^T = K q^T, the whole query in registers), the four maxima meet in LDS, each wave turns ITS scores into weights and leaves them as bf16
// hi + lo; every wave then multiplies all 64 weights with its own quarter of the latent columns.  A share leaves its normalised sums as bf16
// and its (max, sum); k_latent_share_values weights the shares.
#define LAT_KT 32                                  // key tile of the prompt kernel
#define LAT_VS 40                                  // its LDS stride of a transposed column (32 keys + 8)
#define LAD_KT 64                                  // key tile of the decode kernel
#define LAD_VS 72
#define LAD_PS 72                                  // LDS stride of a head's weights
// 4 keys x 8 columns -> column e: the four keys packed
typedef uint32_t u32x4_t __attribute__((ext_vector_type(4)));
__device__ __forceinline__ uint2 column_of(const u32x4_t (&r)[4], int e) {
    const int w = e >> 1;
    const uint32_t sel = (e & 1) ? 0x07060302u : 0x05040100u;        // v_perm: high / low halves of two words
    return make_uint2(__builtin_amdgcn_perm(r[1][w], r[0][w], sel), __builtin_amdgcn_perm(r[3][w], r[2][w], sel));
}
// LDS layouts of the decode kernel, free of bank conflicts for its writes (a wave: 8 keys x 8 chunks) and its fragment reads (16 rows, one chunk):
// a key row is an odd number of 128-byte halves long and its 16-byte chunks are exchanged within groups of 8 by the row's number / 2; the
// 8-byte places of a column row are exchanged in groups of four by the column's number / 16
__host__ __device__ __forceinline__ int lad_key_stride(int CW) { const int k = (CW + 63) / 64 * 64; return k % 128 ? k : k + 64; }
__device__ __forceinline__ int lad_key_at(int row, int chunk, int KS) { return row * KS + ((chunk & ~7) | ((chunk ^ (row >> 1)) & 7)) * 8; }
static size_t latent_decode_lds(const LatentDims& D, int HT) {
    return (size_t)LAD_KT * lad_key_stride(D.CW) * 2 + (size_t)D.Rp * LAD_VS * 2 + (size_t)HT * (2 * 16 * LAD_PS * 2 + 4 * 16 * 4);
}
// NTW: latent tiles per wave (Rp / 64 <= NTW); NST: staging rounds (CW <= 128 HT NST); QF: query fragments (CW / 32 <= QF)
template <int NTW, int NST, int QF, int HT>
__global__ void __launch_bounds__(256 * HT, HT) k_latent_attn_decode(LatentDims D, LatentAttn p, LatentShares sh, int rows) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int KS = lad_key_stride(D.CW);
    bf16_t* sk = reinterpret_cast<bf16_t*>(lds);                                // [64][KS]
    bf16_t* sv = sk + (size_t)LAD_KT * KS;                                      // [Rp][LAD_VS]
    const int tid = threadIdx.x, lane = tid & 63, wave = (tid >> 6) & 3, ht = tid >> 8, li = lane & 15, lq = lane >> 4;
    bf16_t* sw = sv + (size_t)D.Rp * LAD_VS + (size_t)ht * 2 * 16 * LAD_PS;     // [hi, lo][16 heads][LAD_PS]
    float* smx = reinterpret_cast<float*>(sv + (size_t)D.Rp * LAD_VS + (size_t)HT * 2 * 16 * LAD_PS) + ht * 64;      // [4 waves][16 heads]
    const int sp = blockIdx.x / rows, m = blockIdx.x - sp * rows, h0 = (blockIdx.y * HT + ht) * 16;       // (a row's shares on one XCD where rows % 8 == 0)
    const bool on = !p.rows.on || p.rows.on[m];
    const int pos = p.rows.pos[m], seq = p.rows.seq ? p.rows.seq[m] : m;
    const int lo = D.window > 0 ? max(0, pos - D.window + 1) : 0;
    const int nk = pos - lo + 1, per = ((nk + sh.S - 1) / sh.S + 3) & ~3;
    const int k0 = lo + sp * per, k1 = on ? min(k0 + per, pos + 1) : k0;        // this share's keys, in equal tiles of at most LAD_KT
    const int KT = ((per + (per + LAD_KT - 1) / LAD_KT - 1) / ((per + LAD_KT - 1) / LAD_KT) + 3) & ~3;
    const bf16_t* cache = (const bf16_t*)p.cache + (size_t)seq * p.Smax * D.CW;
    const int nch = D.CW >> 3, CT = D.CW >> 5;
    const int kg = ((tid >> 3) & 7) + 8 * ((tid >> 6) & 1), ch0 = (tid & 7) + 8 * (tid >> 7);        // a load of a wave: 8 keys x 128 bytes
    u32x4_t st[NST][4];
    auto fetch = [&](int t) {
        const bf16_t* kr[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) kr[k] = cache + (size_t)min(t + kg + 16 * k, k1 - 1) * D.CW;
#pragma unroll
        for (int i = 0; i < NST; ++i) {
            const int chunk = ch0 + 16 * HT * i;
            if (chunk < nch) {
#pragma unroll
                for (int k = 0; k < 4; ++k) st[i][k] = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(kr[k] + chunk * 8));   // read once per step
            }
        }
    };
    bf16x8_t qf[QF];                                                            // heads past H read head H - 1 and are dropped at the end
    {
        constexpr int NQ = (QF * 4 * 16 + 255) / 256;                           // 16-byte chunks per thread: 16 HT rows x CW / 8 over 256 HT threads
        const bf16_t* q = (const bf16_t*)p.q + (size_t)m * D.H * D.CW;
        const int hb = blockIdx.y * HT * 16;
        u32x4_t qr[NQ];
#pragma unroll
        for (int i = 0; i < NQ; ++i) {
            const int t = min(tid + 256 * HT * i, 16 * HT * nch - 1), r = t / nch, c = t - r * nch;
            qr[i] = *reinterpret_cast<const u32x4_t*>(q + (size_t)min(hb + r, D.H - 1) * D.CW + c * 8);
        }
        __builtin_amdgcn_sched_barrier(0);                                      // loads return in order: the queries are not to wait for the keys
        if (k0 < k1) fetch(k0);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int i = 0; i < NQ; ++i) {
            const int t = tid + 256 * HT * i, r = t / nch, c = t - r * nch;
            if (t < 16 * HT * nch) *reinterpret_cast<u32x4_t*>(sk + lad_key_at(r, c, KS)) = qr[i];
        }
        lds_barrier();
#pragma unroll
        for (int i = 0; i < QF; ++i) {                                          // fragments past the row are zero: the products below need no guards
            const bf16x8_t f = *reinterpret_cast<const bf16x8_t*>(sk + lad_key_at(ht * 16 + li, min(i, CT - 1) * 4 + lq, KS));
            qf[i] = i < CT ? f : (bf16x8_t){0, 0, 0, 0, 0, 0, 0, 0};
        }
        lds_barrier();
    }
    f32x4_t o[NTW];
#pragma unroll
    for (int i = 0; i < NTW; ++i) o[i] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    float mx = -INFINITY, ls = 0.0f;                                            // of head li; ls: this lane's keys only
    for (int t = k0; t < k1; t += KT) {
        const int te = min(t + KT, k1);                                         // end of the tile's keys
#pragma unroll
        for (int i = 0; i < NST; ++i) {
            const int chunk = ch0 + 16 * HT * i;
            if (chunk < nch) {
#pragma unroll
                for (int k = 0; k < 4; ++k) *reinterpret_cast<u32x4_t*>(sk + lad_key_at(kg + 16 * k, chunk, KS)) = st[i][k];
                if (chunk * 8 < D.Rp) {
#pragma unroll
                    for (int e = 0; e < 8; ++e) *reinterpret_cast<uint2*>(sv + (size_t)(chunk * 8 + e) * LAD_VS + 4 * (kg ^ (4 * ((chunk >> 1) & 3)))) = column_of(st[i], e);
                }
            }
        }
        if (te < k1) fetch(te);
        lds_barrier();
        float w[4], tm = -INFINITY;
        {
            f32x4_t s0 = (f32x4_t){0.f, 0.f, 0.f, 0.f}, s1 = s0;
            if (t + wave * 16 < te) {                                           // wave-uniform
                const bf16_t *kr = sk + lad_key_at(wave * 16 + li, lq, KS), *kr1 = sk + lad_key_at(wave * 16 + li, 4 + lq, KS);
#pragma unroll
                for (int i = 0; i < QF; i += 2) {                               // (past the row: its first fragments again, times zero)
                    s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(kr + (i < CT ? i * 32 : 0)), qf[i], s0, 0, 0, 0);
                    s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(kr1 + (i + 1 < CT ? i * 32 : 0)), qf[i + 1], s1, 0, 0, 0);
                }
            }
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                w[e] = t + wave * 16 + lq * 4 + e < te ? (s0[e] + s1[e]) * D.scale : -INFINITY;
                tm = fmaxf(tm, w[e]);
            }
        }
        tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
        tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
        if (lq == 0) smx[wave * 16 + li] = tm;
        lds_barrier();
        const float mn = fmaxf(mx, fmaxf(fmaxf(smx[li], smx[16 + li]), fmaxf(smx[32 + li], smx[48 + li]))), alpha = __expf(mx - mn);
        mx = mn;
        {
            float add = 0.0f;
            bf16_t* pw = sw + (size_t)li * LAD_PS + lq * 16 + wave;             // key 16 wave + kg at place 4 kg + wave, kg = 4 lq + e
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                w[e] = __expf(w[e] - mn);
                add += w[e];
                const bf16_t hi = f32_to_bf16(w[e]);
                pw[4 * e] = hi;
                pw[16 * LAD_PS + 4 * e] = f32_to_bf16(w[e] - bf16_to_f32(hi));
            }
            ls = ls * alpha + add;
        }
        if (t > k0 && __any(alpha != 1.0f)) {                                   // (the first tile has nothing to rescale)
#pragma unroll
            for (int i = 0; i < NTW; ++i) o[i] *= alpha;                        // accumulator column = head li
        }
        lds_barrier();
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            if (ks == 1 && t + 8 >= te) continue;                               // (places 32 .. hold keys kg >= 8: none of them in the share; uniform)
            const bf16x8_t ph = *reinterpret_cast<const bf16x8_t*>(sw + (size_t)li * LAD_PS + ks * 32 + lq * 8),
                           pl = *reinterpret_cast<const bf16x8_t*>(sw + (size_t)(16 + li) * LAD_PS + ks * 32 + lq * 8);
#pragma unroll
            for (int i = 0; i < NTW; ++i) {
                const int tile = min(i * 4 + wave, (D.Rp >> 4) - 1);            // (tiles past the latent repeat its last one and are not stored)
                const bf16x8_t v = lds_frag(sv + (size_t)(tile * 16 + li) * LAD_VS + ((ks * 4 + lq) ^ (2 * (tile & 3))) * 8);
                o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, ph, o[i], 0, 0, 0);        // rows: latent columns, columns: heads
                o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pl, o[i], 0, 0, 0);
            }
        }
        lds_barrier();                                                          // everyone is done with the tile
    }
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
    if (lq == 0) smx[wave * 16 + li] = ls;
    lds_barrier();
    ls = (smx[li] + smx[16 + li]) + (smx[32 + li] + smx[48 + li]);
    if (wave == 0 && lq == 0 && h0 + li < D.H) {
        float* ml = sh.ml + (((size_t)sp * rows + m) * D.H + h0 + li) * 2;
        *reinterpret_cast<float2*>(ml) = make_float2(mx, ls);
    }
    // normalised rows through LDS (the key rows' place), then whole rows
    {
        const float inv = ls > 0.0f ? 1.0f / ls : 0.0f;
        const int OS = D.Rp + 8;
        bf16_t* so = sk + (size_t)ht * 16 * OS;
#pragma unroll
        for (int i = 0; i < NTW; ++i) {
            const int c = (i * 4 + wave) * 16 + lq * 4;
            const float v[4] = {o[i][0] * inv, o[i][1] * inv, o[i][2] * inv, o[i][3] * inv};
            if (c < D.Rp) *reinterpret_cast<uint2*>(so + (size_t)li * OS + c) = pack4_bf16(v);
        }
        lds_barrier();
        bf16_t* out = sh.part + ((size_t)sp * rows + m) * D.H * D.Rp;
#pragma unroll
        for (int r = 0; r < 4; ++r) {                                           // wave w: heads 4 w .. of its tile, a row per step
            const int hd = h0 + wave * 4 + r;
            if (hd < D.H && lane * 8 < D.Rp)
                *reinterpret_cast<u32x4_t*>(out + (size_t)hd * D.Rp + lane * 8) = *reinterpret_cast<const u32x4_t*>(so + (size_t)(wave * 4 + r) * OS + lane * 8);
        }
    }
}

// One block of 8 waves per (head, 8 rows): weights of the shares -> latent sums of the rows (bf16, LDS) -> values.  A wave owns every eighth value
// tile; its weight fragments are requested before the shares are read.
#define LSV_KF 16                                  // k-tiles (Rp <= 512)
#define LSV_ROWS 8
__global__ void __launch_bounds__(512) k_latent_share_values(LatentDims D, LatentShares sh, const bf16_t* __restrict__ uv, size_t uvz, Operand out, int rows) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    bf16_t* so = reinterpret_cast<bf16_t*>(lds);                                // [LSV_ROWS][Rp + 8]
    const int hd = blockIdx.x, m0 = blockIdx.y * LSV_ROWS, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, lq = lane >> 4;
    const int vt = D.vp >> 4, KT = D.Rp >> 5;
    bf16x8_t wf[LSV_KF];
    auto request = [&](int t) {
        const bf16_t* wp = uv + uvz * hd + (size_t)min(t, vt - 1) * KT * 512 + lane * 8;
#pragma unroll
        for (int i = 0; i < LSV_KF; ++i) wf[i] = *reinterpret_cast<const bf16x8_t*>(wp + (size_t)min(i, KT - 1) * 512);
    };
    request(wave);
    const int rc = D.Rp >> 3;
    for (int t = tid; t < LSV_ROWS * rc; t += 512) {
        const int r = t / rc, c = t - r * rc, m = m0 + r;
        bf16x8_t o = {0, 0, 0, 0, 0, 0, 0, 0};
        if (m < rows) {
            const float2* ml = reinterpret_cast<const float2*>(sh.ml) + (size_t)m * D.H + hd;
            const bf16_t* pp = sh.part + ((size_t)m * D.H + hd) * D.Rp + c * 8;
            const size_t ss = (size_t)rows * D.H;
            float a[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f}, l = 0.0f, mx = -INFINITY;
            for (int s0 = 0; s0 < sh.S; s0 += 8) {
                float2 q[8];
                bf16x8_t v[8];
#pragma unroll
                for (int u = 0; u < 8; ++u) {
                    const int s = min(s0 + u, sh.S - 1);
                    q[u] = ml[ss * s];
                    v[u] = *reinterpret_cast<const bf16x8_t*>(pp + ss * s * D.Rp);
                }
                float mn = mx;
#pragma unroll
                for (int u = 0; u < 8; ++u) mn = fmaxf(mn, (s0 + u < sh.S && q[u].y > 0.0f) ? q[u].x : -INFINITY);        // (an empty share holds sum 0)
                const float alpha = mx == -INFINITY ? 0.0f : __expf(mx - mn);
                l *= alpha;
#pragma unroll
                for (int e = 0; e < 8; ++e) a[e] *= alpha;
#pragma unroll
                for (int u = 0; u < 8; ++u) {
                    const float w = (s0 + u < sh.S && q[u].y > 0.0f) ? __expf(q[u].x - mn) * q[u].y : 0.0f;
                    l += w;
#pragma unroll
                    for (int e = 0; e < 8; ++e) a[e] += w * bf16_to_f32((bf16_t)v[u][e]);
                }
                mx = mn;
            }
            const float inv = l > 0.0f ? 1.0f / l : 0.0f;
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = (short)f32_to_bf16(a[e] * inv);
        }
        *reinterpret_cast<bf16x8_t*>(so + (size_t)r * (D.Rp + 8) + c * 8) = o;
    }
    __syncthreads();
    for (int vtile = wave; vtile < vt; vtile += 8) {                            // (no barrier inside)
        if (vtile >= 8) request(vtile);
        f32x4_t a0 = (f32x4_t){0.f, 0.f, 0.f, 0.f}, a1 = a0;
        const bf16_t* xr = so + (size_t)(li & (LSV_ROWS - 1)) * (D.Rp + 8) + lq * 8;       // columns 8 .. 15 of the product repeat the rows, unused
#pragma unroll
        for (int i = 0; i < LSV_KF; i += 2) {
            const bf16x8_t zero = {0, 0, 0, 0, 0, 0, 0, 0};                     // (fragments past the latent: nothing)
            a0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(i < KT ? wf[i] : zero, *reinterpret_cast<const bf16x8_t*>(xr + min(i, KT - 1) * 32), a0, 0, 0, 0);
            a1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(i + 1 < KT ? wf[i + 1] : zero, *reinterpret_cast<const bf16x8_t*>(xr + min(i + 1, KT - 1) * 32), a1, 0, 0, 0);
        }
        const int m = m0 + li, c = vtile * 16 + lq * 4;
        if (li < LSV_ROWS && m < rows) {
            const float v[4] = {a0[0] + a1[0], a0[1] + a1[1], a0[2] + a1[2], a0[3] + a1[3]};
            if (D.v % 4 == 0) {
                if (c < D.v) operand_store4(out, m, hd * D.v + c, v);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) if (c + e < D.v) operand_store1(out, m, hd * D.v + c + e, v[e]);
            }
        }
    }
}

void launch_latent_attn_any(const LatentDims& D, const LatentAttn& p, int rows, hipStream_t s) {
    MIS_REQUIRE(p.rows.pos && p.q && p.cache && p.out && rows >= 1 && D.Rp <= 256 * LAT_OC, MIS_ERR_GENERATION_FAILED, "latent attention: bad operands");
    const size_t sm = (size_t)(D.CW + 256 + 8) * 4;
    if (p.f32) hipLaunchKernelGGL((k_latent_attn_any<float>), dim3(rows, D.H), dim3(256), sm, s, D, p);
    else hipLaunchKernelGGL((k_latent_attn_any<bf16_t>), dim3(rows, D.H), dim3(256), sm, s, D, p);
}
bool latent_decode_mfma_ok(const LatentDims& D) {
    return D.Rp <= 512 && D.CW <= (D.Rp <= 128 ? 256 : D.Rp <= 256 ? 512 : 576) && latent_decode_lds(D, D.H > 16 ? 2 : 1) <= 160 * 1024;
}
// shares per row: at most one block per compute unit (a block fills one), at least 32 keys each
int latent_decode_shares(const LatentDims& D, int rows, int Smax) {
    const char* e = getenv("MIS_LATENT_SHARES");                                // A/B
    const int keys = D.window > 0 ? std::min(D.window, Smax) : Smax, blocks = rows * cdiv(D.H, D.H > 16 ? 32 : 16);
    const int want = e && atoi(e) > 0 ? atoi(e) : std::max(1, 256 / blocks);
    return std::max(1, std::min(std::min(want, cdiv(keys, 32)), 32));
}
void launch_latent_attn_decode(const LatentDims& D, const LatentAttn& p, const LatentShares& sh, int rows, hipStream_t s) {
    MIS_REQUIRE(p.rows.pos && p.q && p.cache && sh.part && sh.ml && sh.S >= 1 && rows >= 1 && !p.f32 && latent_decode_mfma_ok(D), MIS_ERR_GENERATION_FAILED,
                "latent decode attention: bad operands");
    const int HT = D.H > 16 ? 2 : 1;
    const dim3 grid(rows * sh.S, cdiv(D.H, 16 * HT));
    const size_t sm = latent_decode_lds(D, HT);
#define LAT_GO(A, B, C, T)                                                                                                                                      \
    do {                                                                                                                                                        \
        static const hipError_t attr = hipFuncSetAttribute((const void*)k_latent_attn_decode<A, B, C, T>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); \
        HIP_CHECK(attr);                                                                                                                                        \
        hipLaunchKernelGGL((k_latent_attn_decode<A, B, C, T>), grid, dim3(256 * T), sm, s, D, p, sh, rows);                                                     \
    } while (0)
    if (D.Rp <= 128) { if (HT == 1) LAT_GO(2, 2, 8, 1); else LAT_GO(2, 1, 8, 2); }
    else if (D.Rp <= 256) { if (HT == 1) LAT_GO(4, 4, 16, 1); else LAT_GO(4, 2, 16, 2); }
    else { if (HT == 1) LAT_GO(8, 5, 18, 1); else LAT_GO(8, 3, 18, 2); }
#undef LAT_GO
}
void launch_latent_share_values(const LatentDims& D, const LatentShares& sh, const bf16_t* uv, size_t uvz, const Operand& out, int rows, hipStream_t s) {
    MIS_REQUIRE(D.Rp <= 32 * LSV_KF, MIS_ERR_GENERATION_FAILED, "latent values: latent size above 512");
    hipLaunchKernelGGL(k_latent_share_values, dim3(D.H, cdiv(rows, LSV_ROWS)), dim3(512), (size_t)LSV_ROWS * (D.Rp + 8) * 2, s, D, sh, uv, uvz, out, rows);
}

// ============================================================================ expanded attention on the matrix cores (prompts)
// Block = one tile of up to 64 queries of one sequence, one head; wave w owns 16 queries.  Key tiles of 32: key rows [plain | rotary] and transposed
// values go through LDS, fetched one tile ahead.  S^T = K q^T with the key rows permuted (A row i of half f = key 8 (i >> 2) + (i & 3) + 4 f),
// so that a lane's eight scores are eight consecutive keys of ITS query: the weights are the next MFMA's A operand without leaving registers.
template <int KT, int VT>
__global__ void __launch_bounds__(256, 2) k_latent_attn_prefill(LatentDims D, LatentPrefill p) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    const int KS = D.DK + 8;
    bf16_t* sk = reinterpret_cast<bf16_t*>(lds);                                // [32][DK + 8]
    bf16_t* sv = sk + (size_t)LAT_KT * KS;                                      // [vp][LAT_VS]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, lq = lane >> 4, hd = blockIdx.x;
    const LatentTile T = p.tiles[blockIdx.y];
    const int q_last = T.pos0 + T.n - 1;
    const int k_lo = D.window > 0 ? max(T.kpos0, T.pos0 - D.window + 1) : T.kpos0;
    const int ntile = (q_last - k_lo + LAT_KT) / LAT_KT;
    const int kt_n = D.DK >> 5, vt_n = D.vp >> 4;
    constexpr int NK = KT / 2;                                                  // staging rounds of the key rows: 32 DK / 8 / 256 <= KT / 2
    const int nch = D.DK >> 3, nplain = D.np >> 3, nrot = (D.np + D.rp) >> 3, nv = D.vp >> 3;
    int kkey[NK], kch[NK];
#pragma unroll
    for (int i = 0; i < NK; ++i) { const int t = tid + 256 * i; kkey[i] = t / nch; kch[i] = t - kkey[i] * nch; }
    const int vkg = tid & 7, vch = tid >> 3;                                    // 8 groups of 4 keys x vp / 8 chunks (vp <= 256)
    const bf16_t* kplain = p.kv + (size_t)hd * D.np;
    const bf16_t* vals = p.kv + (size_t)D.H * D.np + (size_t)hd * D.vp;
    const bf16_t* crot = p.cache + (size_t)T.seq * p.Smax * D.CW + D.Rp;
    u32x4_t sk_r[NK], sv_r[4];
    auto fetch = [&](int t) {
        const int k0 = k_lo + t * LAT_KT;
#pragma unroll
        for (int i = 0; i < NK; ++i) {
            const int key = min(k0 + min(kkey[i], LAT_KT - 1), q_last);
            const int c = kch[i];
            const bf16_t* src = c < nplain ? kplain + (size_t)(T.krow0 + key - T.kpos0) * p.ldkv + c * 8
                                           : crot + (size_t)key * D.CW + (c < nrot ? c - nplain : 0) * 8;
            sk_r[i] = *reinterpret_cast<const u32x4_t*>(src);
            if (c >= nrot) sk_r[i] = (u32x4_t){0, 0, 0, 0};
        }
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int key = min(k0 + 4 * vkg + k, q_last);
            sv_r[k] = *reinterpret_cast<const u32x4_t*>(vals + (size_t)(T.krow0 + key - T.kpos0) * p.ldkv + min(vch, nv - 1) * 8);
        }
    };
    const int wq0 = wave * 16, qi = wq0 + li;                                   // this lane's query of the tile
    const int qpos = T.pos0 + min(qi, T.n - 1);
    const bool w_on = wq0 < T.n;
    const int w_first = T.pos0 + wq0, w_last = T.pos0 + min(wq0 + 15, T.n - 1);
    bf16x8_t qf[KT];
    {
        const bf16_t* q = p.q + ((size_t)(T.row0 + min(qi, T.n - 1)) * D.H + hd) * D.DK + lq * 8;
#pragma unroll
        for (int i = 0; i < KT; ++i) {                                          // fragments past the row are zero: no guards below
            const bf16x8_t f = *reinterpret_cast<const bf16x8_t*>(q + min(i, kt_n - 1) * 32);
            qf[i] = i < kt_n ? f : (bf16x8_t){0, 0, 0, 0, 0, 0, 0, 0};
        }
    }
    f32x4_t o[VT];
#pragma unroll
    for (int i = 0; i < VT; ++i) o[i] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
    float mx = -INFINITY, ls = 0.0f;
    const int perm = 8 * (li >> 2) + (li & 3);
    fetch(0);
    for (int t = 0; t < ntile; ++t) {
        const int k0 = k_lo + t * LAT_KT;
#pragma unroll
        for (int i = 0; i < NK; ++i)
            if (kkey[i] < LAT_KT) *reinterpret_cast<u32x4_t*>(sk + (size_t)kkey[i] * KS + kch[i] * 8) = sk_r[i];
        if (vch < nv) {
#pragma unroll
            for (int e = 0; e < 8; ++e) *reinterpret_cast<uint2*>(sv + (size_t)(vch * 8 + e) * LAT_VS + 4 * vkg) = column_of(sv_r, e);
        }
        if (t + 1 < ntile) fetch(t + 1);
        lds_barrier();
        if (w_on && k0 <= w_last && (D.window <= 0 || k0 + LAT_KT - 1 > w_first - D.window)) {            // wave-uniform: some key is seen
            f32x4_t s[2];
#pragma unroll
            for (int f = 0; f < 2; ++f) {
                s[f] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
                const bf16_t* kr = sk + (size_t)(perm + 4 * f) * KS + lq * 8;
#pragma unroll
                for (int i = 0; i < KT; ++i)
                    s[f] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(kr + min(i, kt_n - 1) * 32), qf[i], s[f], 0, 0, 0);
            }
            float w[8], tm = -INFINITY;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const int key = k0 + 8 * lq + e;
                const bool seen = key <= qpos && (D.window <= 0 || key > qpos - D.window);
                w[e] = seen ? s[e >> 2][e & 3] * D.scale : -INFINITY;
                tm = fmaxf(tm, w[e]);
            }
            tm = fmaxf(tm, __shfl_xor(tm, 16, 64));
            tm = fmaxf(tm, __shfl_xor(tm, 32, 64));
            const float mn = fmaxf(mx, tm), base = mn == -INFINITY ? 0.0f : mn;  // a query may see none of this tile's keys yet
            const float alpha = __expf(mx - base);
            float add = 0.0f;
#pragma unroll
            for (int e = 0; e < 8; ++e) { w[e] = __expf(w[e] - base); add += w[e]; }
            ls = ls * alpha + add;
            mx = mn;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float aq = __shfl(alpha, lq * 4 + e, 64);
#pragma unroll
                for (int i = 0; i < VT; ++i) o[i][e] *= aq;
            }
            bf16x8_t ph, pl;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const bf16_t hi = f32_to_bf16(w[e]);
                ph[e] = (short)hi;
                pl[e] = (short)f32_to_bf16(w[e] - bf16_to_f32(hi));
            }
#pragma unroll
            for (int i = 0; i < VT; ++i) {
                const bf16x8_t v = lds_frag(sv + (size_t)(min(i, vt_n - 1) * 16 + li) * LAT_VS + lq * 8);        // (tiles past the values are not stored)
                o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ph, v, o[i], 0, 0, 0);
                o[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pl, v, o[i], 0, 0, 0);
            }
        }
        lds_barrier();
    }
    ls += __shfl_xor(ls, 16, 64);
    ls += __shfl_xor(ls, 32, 64);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        const int q = wq0 + lq * 4 + e;
        const float inv = 1.0f / __shfl(ls, lq * 4 + e, 64);
        if (q >= T.n) continue;
        bf16_t* out = p.out + (size_t)(T.row0 + q) * p.ldo + (size_t)hd * D.v;
#pragma unroll
        for (int i = 0; i < VT; ++i) {
            const int c = i * 16 + li;
            if (c < D.v) out[c] = f32_to_bf16(o[i][e] * inv);
        }
    }
}
bool latent_prefill_mfma_ok(const LatentDims& D) { return D.DK <= 256 && D.vp <= 256; }
void launch_latent_attn_prefill(const LatentDims& D, const LatentPrefill& p, hipStream_t s) {
    MIS_REQUIRE(latent_prefill_mfma_ok(D) && p.n_tiles >= 1 && p.ldkv % 8 == 0, MIS_ERR_GENERATION_FAILED, "latent prompt attention: unsupported sizes");
    const dim3 grid(D.H, p.n_tiles);
    const size_t sm = (size_t)LAT_KT * (D.DK + 8) * 2 + (size_t)D.vp * LAT_VS * 2;
    if (D.DK <= 128 && D.vp <= 128) hipLaunchKernelGGL((k_latent_attn_prefill<4, 8>), grid, dim3(256), sm, s, D, p);
    else if (D.DK <= 192 && D.vp <= 128) hipLaunchKernelGGL((k_latent_attn_prefill<6, 8>), grid, dim3(256), sm, s, D, p);
    else hipLaunchKernelGGL((k_latent_attn_prefill<8, 16>), grid, dim3(256), sm, s, D, p);
}
