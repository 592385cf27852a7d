// lm_blocks_mixed.hip - layers that run a mixer, then a feed-forward, each with a norm before it and one behind it (BLOCK_DECAY, BLOCK_PARALLEL of
// lm_blocks.h): weight residency, caches and states, the kernel chain of a decode step and of a prompt pass (kernels: lm_mixers.hip).
//
// Decode step, per layer (bf16): ONE weight-streaming GEMM for everything that reads the layer's norm -> the mixer, which leaves its result as the next
// GEMM's operand (both sides of a parallel mixer side by side along K, their scales multiplied in before the rounding: ONE output product) ->
// split-K slabs -> slabs, norm, residual and the next norm in one launch -> gate | up with silu(gate) up in the epilogue -> down -> residual.
// The norm over a lightning mixer's heads is a factor per row: it waits until behind the output product (the residual launch applies it), the
// mixer only leaves its sums of squares.
#include <math.h>
#include <string.h>
#include <algorithm>
#include "lm_blocks.h"

void LmBlocks::mixed_layer(int li) {
    Layer& l = layers_[li];
    const BlockSpec& b = spec.layers[li];
    auto section = [&](int n) { const int at = l.Nqkv; l.Nqkv += (int)round_up(n, 16); return at; };
    if (l.kind == BLOCK_DECAY) {
        l.S = decay_dims(b.decay.heads, b.decay.dim, b.decay.vdim);
        l.oq = section(l.S.H * l.S.D); l.ok = section(l.S.H * l.S.D); l.ov = section(l.S.H * l.S.E); l.og = section(l.S.H * l.S.E);
        l.Ko = pad_k(l.S.H * l.S.E);
        return;
    }
    const GroupedMixerSpec& g = b.grouped;
    l.A = grouped_dims(g.heads, g.kv_heads, g.dim, g.vdim, g.window, g.keep, g.rot.dims, g.scale, spec.eps);
    l.R = recur_dims(b.recur.width, b.recur.blocks, b.recur.conv);
    l.oq = section(l.A.H * l.A.D); l.ok = section(l.A.G * l.A.D); l.ov = section(l.A.G * l.A.E); l.oy = section(l.R.W); l.ox = section(l.R.W);
    l.KR = (int)round_up(l.A.H * l.A.E, 32);
    l.Ko = pad_k(l.KR + l.R.W);
}

// ============================================================================ weights
void LmBlocks::mixed_tensors(int li, std::vector<std::pair<std::string, std::vector<int64_t>>>& t) const {
    const Layer& l = layers_[li];
    const std::string p = "l" + std::to_string(spec.layers[li].index) + ".", m = p + "mix.";
    const int ff = spec.layers[li].ff;
    t.push_back({p + "norm1", {d}});
    t.push_back({p + "norm1b", {d}});
    if (l.kind == BLOCK_DECAY) {
        const DecayDims& S = l.S;
        t.push_back({m + "q", {S.H * S.D, d}});
        t.push_back({m + "k", {S.H * S.D, d}});
        t.push_back({m + "v", {S.H * S.E, d}});
        t.push_back({m + "g", {S.H * S.E, d}});
        t.push_back({m + "norm", {S.H * S.E}});
        t.push_back({m + "o", {d, S.H * S.E}});
    } else {
        const GroupedDims& A = l.A;
        const RecurDims& R = l.R;
        auto biased = [&](const std::string& n, int N, int K) { t.push_back({n, {N, K}}); t.push_back({n + ".b", {N}}); };
        biased(m + "left.q", A.H * A.D, d);
        biased(m + "left.k", A.G * A.D, d);
        biased(m + "left.v", A.G * A.E, d);
        t.push_back({m + "left.q.norm", {A.D}});
        t.push_back({m + "left.k.norm", {A.D}});
        t.push_back({m + "left.sink", {A.H}});
        biased(m + "left.o", d, A.H * A.E);
        biased(m + "right.y", R.W, d);
        biased(m + "right.x", R.W, d);
        t.push_back({m + "right.conv", {R.W, R.taps}});
        t.push_back({m + "right.conv.b", {R.W}});
        for (const char* n : {"right.ra", "right.ri"}) {
            t.push_back({m + n, {R.B, R.n, R.n}});
            t.push_back({m + n + ".b", {R.B, R.n}});
        }
        t.push_back({m + "right.lam", {R.W}});
        t.push_back({m + "right.o", {d, R.W}});
    }
    if (ff) {
        t.push_back({p + "norm2", {d}});
        t.push_back({p + "norm2b", {d}});
        t.push_back({p + "mlp.gate", {ff, d}});
        t.push_back({p + "mlp.up", {ff, d}});
        t.push_back({p + "mlp.down", {d, ff}});
    }
}

void LmBlocks::mixed_set(int li, const std::string& t, const bf16_t* src, const std::vector<int64_t>& shape, hipStream_t s) {
    const Layer& l = layers_[li];
    Weights& w = *w_[li];
    const int N = (int)shape[0], K = shape.size() > 1 ? (int)shape[1] : 1;
    auto is = [&](const char* n) { return t == n; };
    auto input = [&](int at) {                                                  // rows of the input projections from column `at`
        const int Np = (int)round_up(N, 16);
        place(src, N, K, 1, 0, 1, 1, Np, dp, s);
        pack_rows(w.w1, (size_t)l.Nqkv * dp, Np, dp, at / 16, 1, s);
    };
    auto bias = [&](int at) {
        if (!w.bias1.p) { w.bias1.alloc(l.Nqkv); w.bias1.zero(s); }
        HIP_CHECK(hipMemcpyAsync(w.bias1.p + at, src, (size_t)N * 2, hipMemcpyDeviceToDevice, s));
    };
    auto plain = [&](DevBuf<bf16_t>& dst) {
        size_t n = 1;
        for (int64_t v : shape) n *= (size_t)v;
        dst.alloc(n);
        HIP_CHECK(hipMemcpyAsync(dst.p, src, n * 2, hipMemcpyDeviceToDevice, s));
    };
    auto output = [&](int at) {                                                 // output projection: columns from operand column `at`
        if (!w.wo_rows.p) { w.wo_rows.alloc((size_t)dp * l.Ko); w.wo_rows.zero(s); }
        HIP_CHECK(hipMemcpy2DAsync(w.wo_rows.p + at, (size_t)l.Ko * 2, src, (size_t)K * 2, (size_t)K * 2, N, hipMemcpyDeviceToDevice, s));
        w.wo.alloc((size_t)dp * l.Ko);
        launch_pack_weight(w.wo_rows.p, w.wo.p, dp, l.Ko, dp / 16, 1, 0, s);
    };
    auto blocks = [&](DevBuf<bf16_t>& dst) {                                    // square matrices, packed one after the other
        const RecurDims& R = l.R;
        for (int b = 0; b < R.B; ++b) {
            place(src + (size_t)b * R.n * R.n, R.n, R.n, 1, 0, 1, 1, R.nt * 16, R.np, s);
            pack_rows(dst, (size_t)R.B * R.nt * 16 * R.np, R.nt * 16, R.np, b * R.nt, 1, s);
        }
    };
    if (is("norm1")) norm_row(w.norm1, src, N, dp, s);
    else if (is("norm1b")) norm_row(w.norm1b, src, N, dp, s);
    else if (is("norm2")) norm_row(w.norm2, src, N, dp, s);
    else if (is("norm2b")) norm_row(w.norm2b, src, N, dp, s);
    else if (is("mlp.gate") || is("mlp.up")) {
        place(src, N, K, 1, 0, 1, 1, l.ffp, dp, s);
        pack_rows(w.wgu, (size_t)2 * l.ffp * dp, l.ffp, dp, is("mlp.up") ? 1 : 0, 2, s);
    }
    else if (is("mlp.down")) { place(src, N, K, 1, 0, 1, 1, dp, l.ffp, s); pack_rows(w.wdown, (size_t)dp * l.ffp, dp, l.ffp, 0, 1, s); }
    else if (is("mix.q") || is("mix.left.q")) input(l.oq);
    else if (is("mix.k") || is("mix.left.k")) input(l.ok);
    else if (is("mix.v") || is("mix.left.v")) input(l.ov);
    else if (is("mix.g")) input(l.og);
    else if (is("mix.right.y")) input(l.oy);
    else if (is("mix.right.x")) input(l.ox);
    else if (is("mix.left.q.b")) bias(l.oq);
    else if (is("mix.left.k.b")) bias(l.ok);
    else if (is("mix.left.v.b")) bias(l.ov);
    else if (is("mix.right.y.b")) bias(l.oy);
    else if (is("mix.right.x.b")) { bias(l.ox); x_bias_set_.insert(li); }
    else if (is("mix.o") || is("mix.left.o")) output(0);
    else if (is("mix.right.o")) output(l.KR);
    else if (is("mix.left.o.b")) norm_row(w.bias_o, src, N, dp, s);
    else if (is("mix.norm")) plain(w.mix_norm);
    else if (is("mix.left.q.norm")) plain(w.qn);
    else if (is("mix.left.k.norm")) plain(w.kn);
    else if (is("mix.left.sink")) plain(w.sink);
    else if (is("mix.right.conv")) plain(w.conv);
    else if (is("mix.right.conv.b")) plain(w.conv_b);
    else if (is("mix.right.ra")) blocks(w.ra);
    else if (is("mix.right.ri")) blocks(w.ri);
    else if (is("mix.right.ra.b")) plain(w.ra_b);
    else if (is("mix.right.ri.b")) plain(w.ri_b);
    else if (is("mix.right.lam")) { w.recur_c.alloc(N); launch_softplus_scaled(src, w.recur_c.p, N, 8.0f, s); }
    else throw MisError(MIS_ERR_INVALID_INPUT, "unexpected tensor " + t);
    if (l.kind == BLOCK_PARALLEL && !w.conv32.p && w.conv.p && w.conv_b.p && x_bias_set_.count(li)) {
        const RecurDims& R = l.R;
        w.conv32.alloc((size_t)(R.taps + 2) * R.W);
        launch_conv_tables(w.conv.p, w.conv_b.p, w.bias1.p + l.ox, w.conv32.p, w.conv32.p + (size_t)R.taps * R.W, w.conv32.p + (size_t)(R.taps + 1) * R.W, R.W, R.taps, s);
    }
    if (l.kind == BLOCK_DECAY && !w.decay.p) {
        const std::vector<float>& c = spec.layers[li].decay.decay;
        w.decay.alloc(c.size());
        HIP_CHECK(hipMemcpyAsync(w.decay.p, c.data(), c.size() * 4, hipMemcpyHostToDevice, s));
        HIP_CHECK(hipStreamSynchronize(s));
    }
}
double LmBlocks::mixed_weight_bytes(int li) const {
    const Layer& l = layers_[li];
    const double ff = 3.0 * d * spec.layers[li].ff;
    if (l.kind == BLOCK_DECAY) return 2.0 * (ff + (double)d * (2.0 * l.S.H * l.S.D + 3.0 * l.S.H * l.S.E));
    const GroupedDims& A = l.A;
    return 2.0 * (ff + (double)d * ((A.H + A.G) * A.D + (A.H + A.G) * A.E + 3.0 * l.R.W) + 2.0 * l.R.W * l.R.n);
}

// ============================================================================ caches, states, buffers
void LmBlocks::mixed_reset(int li, hipStream_t s) {
    Layer& l = layers_[li];
    const int max_s = dp > 8192 ? 4 : 8;                                       // slabs the residual kernel takes
    l.s1 = l.s2 = 1;
    if (!f32) {
        l.s1 = std::min(max_s, gemm_choose_split(dp / 16 / 2, l.Ko / 32, 4, max_s));
        if (l.ffp) l.s2 = std::min(max_s, gemm_choose_split(dp / 16 / 2, l.ffp / 32, 4, max_s));
    }
    if (l.kind == BLOCK_DECAY) { state_[li]->alloc((size_t)batch_ * l.S.H * l.S.D * l.S.Es); return; }
    l.shares = !f32 && grouped_mfma_ok(l.A) ? grouped_decode_shares(l.A, batch_, Smax_) : 1;
    // a masked value still enters the matrix cores, times zero: it has to be a number
    cache_[li]->alloc((size_t)batch_ * l.A.G * Smax_ * (l.A.Dp + l.A.Ep) * esz());
    cache_[li]->zero(s);
    state_[li]->alloc((size_t)batch_ * (1 + l.R.taps) * l.R.W);
}
void LmBlocks::mixed_buffers(MixBuffers& b, int rows, hipStream_t s) {
    size_t n_u = 0, n_raw = 0, n_ss = 0, n_ff = 0, n_part = 0;
    bool mixed = false;
    for (auto& l : layers_) {
        if (l.kind == BLOCK_LATENT) continue;
        mixed = true;
        if (f32) { n_u = std::max(n_u, (size_t)l.R.B * l.R.np); n_raw = std::max(n_raw, (size_t)l.R.B * l.R.nt * 16); }
        else if (&b == &pmix_) n_u = n_raw = std::max(n_u, (size_t)l.R.W);      // local states, decays, carried states
        n_ss = std::max(n_ss, (size_t)l.S.H * l.S.ns); n_ff = std::max(n_ff, (size_t)l.ffp);
        if (&b == &mix_ && l.shares > 1) n_part = std::max(n_part, (size_t)l.shares * batch_ * l.A.H * l.A.Ep);
    }
    if (!mixed) return;
    const bool grow = b.ss.n < rows * std::max<size_t>(n_ss, 1);
    b.u.alloc(rows * n_u); b.raw_r.alloc(rows * n_raw); b.raw_g.alloc(rows * n_raw); b.ss.alloc(rows * n_ss);
    if (f32) b.gu.alloc(rows * 2 * n_ff);
    b.part.alloc(&b == &pmix_ ? (size_t)rows * dp : n_part);
    if (grow) b.ss.zero(s);
}

// ============================================================================ mixers
void LmBlocks::mixer(int li, const float* proj, void* q, const Operand& out, const MixRows& r, MixBuffers& b, hipStream_t s) {
    const Layer& l = layers_[li];
    const Weights& w = W(li);
    if (l.kind == BLOCK_DECAY) {
        DecayParams p{};
        p.proj = proj; p.ld = l.Nqkv; p.oq = l.oq; p.ok = l.ok; p.ov = l.ov; p.og = l.og;
        p.decay = w.decay.p; p.norm = w.mix_norm.p; p.spans = r.spans; p.state = state_[li]->p; p.out = out; p.ss = b.ss.p;
        if (f32 || !decay_mfma_ok(l.S)) launch_decay_any(l.S, p, r.n_spans, s);
        else if (!r.spans.span) launch_decay_step(l.S, p, r.M, s);
        else { p.act = reinterpret_cast<const bf16_t*>(proj); launch_decay_prefill(l.S, p, r.segs, r.n_segs, r.n_segs > r.n_spans, b.ends.p, s); }
        return;
    }
    const GroupedDims& A = l.A;
    const RecurDims& R = l.R;
    uint8_t* kc = cache_[li]->p;
    uint8_t* vc = kc + (size_t)batch_ * A.G * Smax_ * A.Dp * esz();
    GroupedRows gr{};
    gr.proj = proj; gr.ld = l.Nqkv; gr.oq = l.oq; gr.ok = l.ok; gr.ov = l.ov; gr.bias = w.bias1.p; gr.qn = w.qn.p; gr.kn = w.kn.p;
    gr.rope_cos = ropes_[l.rope].cs.p; gr.rope_sin = ropes_[l.rope].sn.p; gr.rows = r.rows; gr.kc = kc; gr.vc = vc; gr.Smax = Smax_; gr.q = q; gr.f32 = f32;
    GroupedAttn ga{};
    ga.q = q; ga.kc = kc; ga.vc = vc; ga.Smax = Smax_; ga.sink = w.sink.p; ga.rows = r.rows; ga.out = out; ga.out_scale = spec.layers[li].left_scale; ga.f32 = f32;
    RecurParams p{};
    p.proj = proj; p.ld = l.Nqkv; p.oy = l.oy; p.ox = l.ox; p.bias = w.bias1.p; p.conv = w.conv.p; p.conv_b = w.conv_b.p; p.ra_b = w.ra_b.p; p.ri_b = w.ri_b.p;
    p.c = w.recur_c.p; p.rows = r.rows; p.pos0 = r.pos0; p.spans = r.spans; p.state = state_[li]->p; p.hist = state_[li]->p + (size_t)batch_ * R.W;
    p.out = out; p.col0 = l.KR; p.out_scale = spec.layers[li].right_scale;
    const bool mfma = !f32 && grouped_mfma_ok(A), step = !r.spans.span;
    if (!f32) { p.ra = w.ra.p; p.ri = w.ri.p; p.conv_t = w.conv32.p; p.conv_b32 = w.conv32.p + (size_t)R.taps * R.W; p.bias_x = p.conv_b32 + R.W; }
    if (mfma && step) {                                                        // both sides in one launch
        GroupedShares sh;
        sh.S = l.shares; sh.part = b.part.p; sh.ml = share_ml_.p;
        launch_grouped_attn_decode(A, gr, ga, sh, &R, &p, r.M, s);
        return;
    }
    if (mfma) launch_grouped_rows_prefill(A, gr, r.tiles, r.n_tiles, r.M, s);
    else launch_grouped_rows(A, gr, r.M, s);
    if (mfma) launch_grouped_attn_prefill(A, ga, r.tiles, r.n_tiles, s);
    else launch_grouped_attn_any(A, ga, r.M, s);
    if (!f32) {
        if (step) launch_recur_step(R, p, r.M, s);
        else launch_recur_prefill(R, p, r.chunks, r.n_chunks, b.u.p, b.raw_r.p, b.raw_g.p, s);
        return;
    }
    launch_conv_rows(R, p, b.u.p, r.M, s);
    GemmF32 g{};
    g.X = b.u.p; g.ldx = R.B * R.np; g.xz = R.np; g.wz = (size_t)R.nt * 16 * R.np; g.ldo = R.B * R.nt * 16; g.oz = R.nt * 16;
    g.M = r.M; g.NT = R.nt; g.KT = R.np / 32; g.n_valid = R.nt * 16; g.heads = R.B;
    g.W = w.ra.p; g.out = b.raw_r.p;
    launch_gemm_f32(g, s);
    g.W = w.ri.p; g.out = b.raw_g.p;
    launch_gemm_f32(g, s);
    launch_gated_scan_any(R, p, b.u.p, b.raw_r.p, b.raw_g.p, r.n_spans, s);
}

static SublayerOut mixer_out(const float* part, int S, bool decay, const DecayDims& D, const float* ss, const bf16_t* bias, float scale) {
    SublayerOut y;
    y.p = part; y.S = S;
    if (decay) { y.ss = ss; y.n_ss = D.H * D.ns; y.ss_cols = D.H * D.E; }
    else { y.bias = bias; y.bias_scale = scale; }
    return y;
}

// ============================================================================ decode step
void LmBlocks::mixed_step_layer(int li, const BlockRows& r, hipStream_t s) {
    const Layer& l = layers_[li];
    const Weights& w = W(li);
    void* at = attn_[columns(li)].p;
    const int rows = f32 ? batch_ : Mpad_;
    auto skinny = [&](const bf16_t* Wp, const void* X, float* out, int NT, int KT, int S, int N) {
        const bool wide = S == 1 && Mpad_ <= 32 && NT / 4 >= 192;              // four n-tiles per wave where the launch still fills the chip
        const bool pairs = wide || (KT >= 64 && Mpad_ <= 32);                  // two waves per item instead of four
        launch_gemm_skinny(EPI_PARTIAL, wide ? 4 : 2, pairs ? 2 : 4, Wp, (const bf16_t*)X, out, NT, KT, S, N, Mpad_, s, nullptr, wide ? 2 : 4);
    };
    if (f32) launch_gemm_f32(gemm32(h_.p, dp, w.w1.p, qkv_.p, l.Nqkv, batch_, l.Nqkv, dp, F32_STORE), s);
    else skinny(w.w1.p, h_.p, qkv_.p, l.Nqkv / 16, dp / 32, 1, l.Nqkv);
    MixRows mr;
    mr.rows.pos = r.pos_cur; mr.rows.on = r.active; mr.pos0 = nullptr; mr.spans.pos = r.pos_cur; mr.spans.on = r.active; mr.M = mr.n_spans = batch_;
    mixer(li, qkv_.p, q_.p, operand(at, l.Ko, Mpad_, true), mr, mix_, s);
    if (f32) launch_gemm_f32(gemm32(at, l.Ko, w.wo.p, part_.p, dp, batch_, dp, l.Ko, F32_STORE), s);
    else skinny(w.wo.p, at, part_.p, dp / 16, l.Ko / 32, l.s1, dp);
    const SublayerOut y1 = mixer_out(part_.p, l.s1, l.kind == BLOCK_DECAY, l.S, mix_.ss.p, w.bias_o.p, spec.layers[li].left_scale);
    launch_post_norm_residual(y1, Mpad_, x_.p, w.norm1b.p, l.ffp ? w.norm2.p : norm_after(li), spec.norm_add, operand(h_.p, dp, Mpad_, true), d, dp, spec.eps, rows, s);
    if (!l.ffp) return;
    if (f32) {
        launch_gemm_f32(gemm32(h_.p, dp, w.wgu.p, mix_.gu.p, 2 * l.ffp, batch_, 2 * l.ffp, dp, F32_STORE), s);
        launch_swiglu_rows_f32(mix_.gu.p, 2 * l.ffp, (float*)act_.p, l.ffp, l.ffp, batch_, s);
        launch_gemm_f32(gemm32(act_.p, l.ffp, w.wdown.p, part_.p, dp, batch_, dp, l.ffp, F32_STORE), s);
    } else {
        const int NT = l.ffp / 8;
        const bool wide = Mpad_ <= 32 && NT / 4 >= 192;
        launch_gemm_skinny(EPI_SWIGLU, wide ? 4 : 2, 4, w.wgu.p, (const bf16_t*)h_.p, act_.p, NT, dp / 32, 1, l.ffp, Mpad_, s);
        skinny(w.wdown.p, act_.p, part_.p, dp / 16, l.ffp / 32, l.s2, dp);
    }
    SublayerOut y2;
    y2.p = part_.p; y2.S = l.s2;
    launch_post_norm_residual(y2, Mpad_, x_.p, w.norm2b.p, norm_after(li), spec.norm_add, operand(h_.p, dp, Mpad_, true), d, dp, spec.eps, rows, s);
}

// ============================================================================ prompt pass
void LmBlocks::mixed_pass_layer(int li, const MixRows& r, hipStream_t s) {
    const Layer& l = layers_[li];
    const Weights& w = W(li);
    void* at = pattn_[columns(li)].p;
    const int M = r.M;
    auto product = [&](const void* X, const bf16_t* Wp, float* out, int N, int K) {
        if (f32) launch_gemm_f32(gemm32(X, K, Wp, out, N, M, N, K, F32_STORE), s);
        else launch_gemm_pf(PF_F32, (const bf16_t*)X, Wp, out, M, N, K, s);
    };
    const Operand h = operand(ph_.p, dp, 0, false);
    if (!f32 && l.kind == BLOCK_DECAY && decay_mfma_ok(l.S)) {
        PfExtra ex; ex.ldc = l.Nqkv; ex.split = l.og / 16;
        launch_gemm_pf(PF_ACT_ROWS, (const bf16_t*)ph_.p, w.w1.p, pqkv_.p, M, l.Nqkv, dp, s, ex);
    } else product(ph_.p, w.w1.p, pqkv_.p, l.Nqkv, dp);
    mixer(li, pqkv_.p, pq_.p, operand(at, l.Ko, 0, false), r, pmix_, s);
    product(at, w.wo.p, pmix_.part.p, dp, l.Ko);
    const SublayerOut y1 = mixer_out(pmix_.part.p, 1, l.kind == BLOCK_DECAY, l.S, pmix_.ss.p, w.bias_o.p, spec.layers[li].left_scale);
    launch_post_norm_residual(y1, M, px_.p, w.norm1b.p, l.ffp ? w.norm2.p : norm_after(li), spec.norm_add, h, d, dp, spec.eps, M, s);
    if (!l.ffp) return;
    if (f32) {
        product(ph_.p, w.wgu.p, pmix_.gu.p, 2 * l.ffp, dp);
        launch_swiglu_rows_f32(pmix_.gu.p, 2 * l.ffp, (float*)pact_.p, l.ffp, l.ffp, M, s);
    } else launch_gemm_pf(PF_SWIGLU, (const bf16_t*)ph_.p, w.wgu.p, pact_.p, M, 2 * l.ffp, dp, s);
    product(pact_.p, w.wdown.p, pmix_.part.p, dp, l.ffp);
    SublayerOut y2;
    y2.p = pmix_.part.p;
    launch_post_norm_residual(y2, M, px_.p, w.norm2b.p, norm_after(li), spec.norm_add, h, d, dp, spec.eps, M, s);
}
