// lm_blocks.hip - host side of the layer-list language models: configuration, weight residency, caches, the kernel chain of a decode step and of
// a prompt pass (see lm_blocks.h; kernels: lm_latent.hip, GEMMs: lm_kernels.hip / lm_prefill.hip).
//
// Decode step, per layer (bf16): ONE weight-streaming GEMM for everything that reads the layer's norm - queries, latent, rotary key (float32
// sums) and the feed-forward's up rows (relu^2 in the epilogue, packed for the down projection) -> latent row + absorbed queries (one launch)
// -> attention over the latent cache in shares of keys -> shares weighted, values -> both projections back to the width as split-K slabs of ONE
// launch -> x += ls1 sum + ls2 sum, norm for the next layer.  The residual stream, scores, norms and rotations are float32.
// Prompt pass: rows = tokens of all requests, (sequence, position) per row; k_gemm_pf GEMMs, keys and values expanded from the latent
// cache for the chunk's keys and the window before it, both projections added to the stream in their epilogues.
// Layers that run one sublayer after the other (BLOCK_DECAY, BLOCK_PARALLEL): lm_blocks_mixed.hip.
#include <math.h>
#include <string.h>
#include <algorithm>
#include "lm_blocks.h"

// ============================================================================ configuration
bool block_architecture_known(const std::string& name) { return name == "Rugunex" || name == "Vamunex"; }

static const JsonValue& need(const JsonValue& o, const char* key, const char* where) {
    const JsonValue* v = o.get(key);
    MIS_REQUIRE(v && v->type != JsonValue::NUL, MIS_ERR_INVALID_INPUT, "config.json: %s has no '%s'", where, key);
    return *v;
}
static double need_num(const JsonValue& o, const char* key, const char* where) {
    const JsonValue& v = need(o, key, where);
    MIS_REQUIRE(v.type == JsonValue::NUM, MIS_ERR_INVALID_INPUT, "config.json: '%s' of %s is not a number", key, where);
    return v.num;
}
static LatentMixerSpec parse_latent_mixer(const JsonValue& m) {
    LatentMixerSpec x;
    x.heads = (int)need_num(m, "heads", "mixer");
    x.dim = (int)need_num(m, "dim", "mixer");
    x.rot_dim = (int)need_num(m, "rot_dim", "mixer");
    x.vdim = (int)need_num(m, "vdim", "mixer");
    x.kv_rank = (int)need_num(m, "kv_rank", "mixer");
    x.scale = (float)need_num(m, "scale", "mixer");
    const JsonValue* mask = m.get("mask");
    if (mask && mask->type == JsonValue::OBJ) x.window = (int)mask->number_or("size", 0);
    const JsonValue& rot = need(m, "rot", "mixer");
    x.rot.dims = (int)need_num(rot, "dims", "rot");
    x.rot.base = need_num(rot, "base", "rot");
    if (const JsonValue* sc = rot.get("scaling"))
        if (sc->type == JsonValue::OBJ) {
            x.rot.yarn = true;
            x.rot.factor = need_num(*sc, "factor", "rot.scaling");
            x.rot.original = need_num(*sc, "original", "rot.scaling");
            x.rot.fast = need_num(*sc, "fast", "rot.scaling");
            x.rot.slow = need_num(*sc, "slow", "rot.scaling");
        }
    MIS_REQUIRE(x.heads >= 1 && x.dim >= 1 && x.rot_dim >= 1 && x.vdim >= 1 && x.kv_rank >= 1 && x.kv_rank <= 2048 && x.window >= 0, MIS_ERR_INVALID_INPUT,
                "latent attention: bad sizes");
    MIS_REQUIRE(x.rot.dims >= 0 && x.rot.dims % 2 == 0 && x.rot.dims <= x.rot_dim && x.rot.base > 0, MIS_ERR_INVALID_INPUT, "latent attention: bad rotary sizes");
    return x;
}
static RotarySpec parse_rotary(const JsonValue& m) {
    RotarySpec r;
    const JsonValue* rot = m.get("rot");
    if (!rot || rot->type != JsonValue::OBJ) return r;
    r.dims = (int)need_num(*rot, "dims", "rot");
    r.base = need_num(*rot, "base", "rot");
    return r;
}
static GroupedMixerSpec parse_grouped_mixer(const JsonValue& m) {
    GroupedMixerSpec x;
    x.heads = (int)need_num(m, "heads", "mixer");
    x.kv_heads = (int)need_num(m, "kv_heads", "mixer");
    x.dim = (int)need_num(m, "dim", "mixer");
    x.vdim = (int)need_num(m, "vdim", "mixer");
    x.scale = (float)need_num(m, "scale", "mixer");
    const JsonValue* mask = m.get("mask");
    if (mask && mask->type == JsonValue::OBJ) {
        x.window = (int)mask->number_or("size", 0);
        x.keep = (int)mask->number_or("keep_first", 0);
    }
    x.rot = parse_rotary(m);
    MIS_REQUIRE(x.heads >= 1 && x.kv_heads >= 1 && x.heads % x.kv_heads == 0 && x.dim >= 1 && x.vdim >= 1 && x.window >= 0 && x.keep >= 0, MIS_ERR_INVALID_INPUT,
                "grouped attention: bad sizes");
    MIS_REQUIRE(x.rot.dims >= 0 && x.rot.dims % 2 == 0 && x.rot.dims <= x.dim && x.rot.base > 0, MIS_ERR_INVALID_INPUT, "grouped attention: bad rotary sizes");
    return x;
}
static RecurMixerSpec parse_recur_mixer(const JsonValue& m) {
    RecurMixerSpec x;
    x.width = (int)need_num(m, "width", "mixer");
    x.blocks = (int)need_num(m, "blocks", "mixer");
    x.conv = (int)need_num(m, "conv", "mixer");
    MIS_REQUIRE(x.width >= 1 && x.blocks >= 1 && x.width % x.blocks == 0 && x.conv >= 1, MIS_ERR_INVALID_INPUT, "gated recurrence: bad sizes");
    return x;
}
static DecayMixerSpec parse_decay_mixer(const JsonValue& m) {
    DecayMixerSpec x;
    x.heads = (int)need_num(m, "heads", "mixer");
    x.dim = (int)need_num(m, "dim", "mixer");
    x.vdim = (int)need_num(m, "vdim", "mixer");
    const JsonValue& d = need(m, "decay", "mixer");
    MIS_REQUIRE(x.heads >= 1 && x.dim >= 1 && x.vdim >= 1, MIS_ERR_INVALID_INPUT, "lightning attention: bad sizes");
    MIS_REQUIRE(d.type == JsonValue::ARR && (int)d.arr.size() == x.heads, MIS_ERR_INVALID_INPUT, "lightning attention: 'decay' needs one number per head");
    for (auto& v : d.arr) {
        MIS_REQUIRE(v.type == JsonValue::NUM && v.num >= 0.0 && v.num <= 1.0, MIS_ERR_INVALID_INPUT, "lightning attention: 'decay' outside 0 .. 1");
        x.decay.push_back((float)v.num);
    }
    return x;
}
// the feed-forward's width (0: none)
static int parse_mlp(const JsonValue& layer, int i) {
    const JsonValue* mlp = layer.get("mlp");
    if (!mlp || mlp->type != JsonValue::OBJ) return 0;
    const JsonValue* kind = mlp->get("kind");
    MIS_REQUIRE(!kind || (kind->type == JsonValue::STR && kind->str == "dense"), MIS_ERR_INVALID_INPUT, "layer %d: unknown feed-forward kind", i);
    const int ff = (int)need_num(*mlp, "ff", "mlp");
    MIS_REQUIRE(ff >= 1, MIS_ERR_INVALID_INPUT, "layer %d: bad feed-forward size", i);
    return ff;
}
static const std::string& layer_type(const JsonValue& e, int i) {
    const JsonValue& type = need(e, "type", "a layer");
    MIS_REQUIRE(type.type == JsonValue::STR, MIS_ERR_INVALID_INPUT, "layer %d: 'type' is not a string", i);
    return type.str;
}
static void parse_rugunex_layers(const JsonValue& ls, BlockModelSpec& sp) {
    for (size_t i = 0; i < ls.arr.size(); ++i) {
        const JsonValue& e = ls.arr[i];
        const std::string& type = layer_type(e, (int)i);
        MIS_REQUIRE(type == "latent_attention", MIS_ERR_INVALID_INPUT, "layer %d: unknown type '%s'", (int)i, type.c_str());
        BlockSpec b;
        b.index = (int)i;
        b.mix = parse_latent_mixer(need(e, "mixer", "a layer"));
        b.ff = parse_mlp(e, (int)i);
        const JsonValue* wo = e.get("weights_of");
        if (!wo && e.get("mixer")) wo = e.get("mixer")->get("weights_of");
        if (wo && wo->type == JsonValue::NUM) {
            b.weights_of = (int)wo->num;
            MIS_REQUIRE(b.weights_of >= 0 && b.weights_of < (int)ls.arr.size() && b.weights_of != (int)i, MIS_ERR_INVALID_INPUT, "layer %d: bad weights_of", (int)i);
        }
        sp.layers.push_back(b);
    }
    for (size_t i = 0; i < sp.layers.size(); ++i) {                           // chains of references end at a layer that owns its tensors
        int o = (int)i, hops = 0;
        while (sp.layers[o].weights_of >= 0 && hops++ <= (int)sp.layers.size()) o = sp.layers[o].weights_of;
        MIS_REQUIRE(sp.layers[o].weights_of < 0, MIS_ERR_INVALID_INPUT, "layer %d: weights_of runs in a circle", (int)i);
        if (o == (int)i) continue;
        const LatentMixerSpec &x = sp.layers[i].mix, &y = sp.layers[o].mix;
        MIS_REQUIRE(x.heads == y.heads && x.dim == y.dim && x.rot_dim == y.rot_dim && x.vdim == y.vdim && x.kv_rank == y.kv_rank && sp.layers[i].ff == sp.layers[o].ff,
                    MIS_ERR_INVALID_INPUT, "layer %d: sizes differ from those of the layer whose weights it uses", (int)i);
        sp.layers[i].weights_of = o;
    }
}
static void parse_vamunex_layers(const JsonValue& j, const JsonValue& ls, BlockModelSpec& sp) {
    const int n = (int)ls.arr.size();
    std::vector<BlockSpec> one;
    for (int i = 0; i < n; ++i) {
        const JsonValue& e = ls.arr[i];
        const std::string& type = layer_type(e, i);
        const JsonValue& m = need(e, "mixer", "a layer");
        BlockSpec b;
        b.index = i;
        if (type == "lightning") {
            b.kind = BLOCK_DECAY;
            b.decay = parse_decay_mixer(m);
        } else {
            MIS_REQUIRE(type == "parallel", MIS_ERR_INVALID_INPUT, "layer %d: unknown type '%s'", i, type.c_str());
            b.kind = BLOCK_PARALLEL;
            b.grouped = parse_grouped_mixer(need(m, "left", "mixer"));
            b.recur = parse_recur_mixer(need(m, "right", "mixer"));
            b.left_scale = (float)need_num(m, "left_scale", "mixer");
            b.right_scale = (float)need_num(m, "right_scale", "mixer");
        }
        b.ff = parse_mlp(e, i);
        one.push_back(b);
    }
    int start = 0, stop = 0, times = 1;
    if (const JsonValue* lp = j.get("loop"))
        if (lp->type == JsonValue::OBJ) {
            start = (int)need_num(*lp, "start", "loop"); stop = (int)need_num(*lp, "stop", "loop"); times = (int)need_num(*lp, "times", "loop");
            MIS_REQUIRE(start >= 0 && start <= stop && stop <= n && times >= 1, MIS_ERR_INVALID_INPUT, "config.json: bad 'loop'");
        }
    std::vector<int> first(n, -1);
    auto run = [&](int i) {
        BlockSpec b = one[i];
        b.weights_of = first[i];
        if (first[i] < 0) first[i] = (int)sp.layers.size();
        sp.layers.push_back(b);
    };
    for (int i = 0; i < start; ++i) run(i);
    for (int t = 0; t < times; ++t) for (int i = start; i < stop; ++i) run(i);
    for (int i = stop; i < n; ++i) run(i);
}
BlockModelSpec parse_block_model(const JsonValue& j) {
    MIS_REQUIRE(j.type == JsonValue::OBJ, MIS_ERR_INVALID_INPUT, "config.json is not an object");
    BlockModelSpec sp;
    const JsonValue& a = need(j, "architecture", "the model");
    MIS_REQUIRE(a.type == JsonValue::STR && block_architecture_known(a.str), MIS_ERR_INVALID_INPUT, "unknown architecture '%s'", a.str.c_str());
    sp.architecture = a.str;
    sp.width = (int)need_num(j, "width", "the model");
    sp.vocab = (int)need_num(j, "vocab", "the model");
    sp.eps = (float)need_num(need(j, "norm", "the model"), "eps", "norm");
    MIS_REQUIRE(sp.width >= 1 && sp.width <= 16384 && sp.vocab >= 1, MIS_ERR_INVALID_INPUT, "bad model width or vocabulary");
    const JsonValue& ls = need(j, "layers", "the model");
    MIS_REQUIRE(ls.type == JsonValue::ARR && !ls.arr.empty(), MIS_ERR_INVALID_INPUT, "config.json: 'layers' is empty");
    if (sp.architecture == "Vamunex") {
        sp.embed_norm = false;
        sp.norm_add = 1.0f;
        parse_vamunex_layers(j, ls, sp);
    } else {
        sp.logit_scale = (float)j.number_or("logit_scale", 1.0);
        sp.softcap = (float)j.number_or("logit_softcap", 0.0);
        parse_rugunex_layers(ls, sp);
    }
    return sp;
}

int pad_k(int k) { return std::max(128, (int)round_up(k, 64)); }        // K of a GEMM operand (k_gemm_pf: whole 64-column steps, two at least)

LmBlocks::LmBlocks(const BlockModelSpec& sp, bool f32_) : spec(sp), f32(f32_) {
    d = sp.width; dp = pad_k(d); V = sp.vocab; Vpad = (int)round_up(V, 16); L = (int)sp.layers.size();
    for (int i = 0; i < L; ++i) {
        const BlockSpec& b = sp.layers[i];
        Layer l{};
        l.kind = b.kind;
        l.owner = b.weights_of >= 0 ? b.weights_of : i;
        l.ffp = b.ff > 0 ? pad_k(b.ff) : 0;
        const RotarySpec& rot = b.kind == BLOCK_PARALLEL ? b.grouped.rot : b.mix.rot;
        for (l.rope = 0; l.rope < (int)ropes_.size() && !(ropes_[l.rope].spec == rot); ++l.rope) {}
        if (l.rope == (int)ropes_.size()) { ropes_.emplace_back(); ropes_.back().spec = rot; }
        w_.emplace_back(b.weights_of >= 0 ? nullptr : new Weights());
        if (b.kind != BLOCK_LATENT) {
            layers_.push_back(l);
            mixed_layer(i);
            continue;
        }
        l.D = latent_dims(b.mix.heads, b.mix.dim, b.mix.rot_dim, b.mix.vdim, b.mix.kv_rank, b.mix.window, b.mix.rot.dims, b.mix.scale, sp.eps);
        l.Nqkv = l.D.H * (l.D.np + l.D.rp) + l.D.Rp + l.D.rp;
        l.Ko = pad_k(l.D.H * l.D.v);
        layers_.push_back(l);
    }
}

// ============================================================================ weights
// dst [Np][Kp] (zero padded) from src [N][K]: source rows come in groups of part1 + part2; a group's first part goes to dst row g * g_out, its
// second to g * g_out + off2
__global__ void k_place_rows(const bf16_t* __restrict__ src, bf16_t* __restrict__ dst, int N, int K, int part1, int part2, int g_out, int off2, int Np, int Kp) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (size_t)Np * Kp) return;
    const int n = (int)(i / Kp), k = (int)(i - (size_t)n * Kp), g = n / g_out, o = n - g * g_out;
    int src_n = -1;
    if (o < part1) src_n = g * (part1 + part2) + o;
    else if (o >= off2 && o - off2 < part2) src_n = g * (part1 + part2) + part1 + (o - off2);
    dst[i] = (src_n >= 0 && src_n < N && k < K) ? src[(size_t)src_n * K + k] : (bf16_t)0;
}
// W_uk [H n][R] -> per head transposed [H][Rp][np]
__global__ void k_place_head_transposed(const bf16_t* __restrict__ src, bf16_t* __restrict__ dst, int H, int n, int R, int Rp, int np) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (size_t)H * Rp * np) return;
    const int j = (int)(i % np), rr = (int)((i / np) % Rp), h = (int)(i / ((size_t)np * Rp));
    dst[i] = (j < n && rr < R) ? src[((size_t)h * n + j) * R + rr] : (bf16_t)0;
}
void LmBlocks::place(const bf16_t* src, int64_t N, int64_t K, int part1, int part2, int g_out, int off2, int Np, int Kp, hipStream_t s) {
    const size_t n = (size_t)Np * Kp;
    place_.alloc(n);
    hipLaunchKernelGGL(k_place_rows, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, src, place_.p, (int)N, (int)K, part1, part2, g_out, off2, Np, Kp);
}

std::vector<std::pair<std::string, std::vector<int64_t>>> LmBlocks::tensor_list() const {
    std::vector<std::pair<std::string, std::vector<int64_t>>> t = {{"embed", {V, d}}, {"final.norm", {d}}, {"head", {V, d}}};
    if (spec.embed_norm) t.push_back({"embed.norm", {d}});
    for (int i = 0; i < L; ++i) {
        if (layers_[i].owner != i) continue;
        if (layers_[i].kind != BLOCK_LATENT) { mixed_tensors(i, t); continue; }
        const LatentDims& D = layers_[i].D;
        const std::string p = "l" + std::to_string(i) + ".";
        const int ff = spec.layers[i].ff;
        t.push_back({p + "norm1", {d}});
        t.push_back({p + "mix.q", {D.H * (D.n + D.r), d}});
        t.push_back({p + "mix.dkv", {D.R + D.r, d}});
        t.push_back({p + "mix.dkv.norm", {D.R}});
        t.push_back({p + "mix.uk", {D.H * D.n, D.R}});
        t.push_back({p + "mix.uv", {D.H * D.v, D.R}});
        t.push_back({p + "mix.o", {d, D.H * D.v}});
        t.push_back({p + "ls1", {d}});
        if (ff) {
            t.push_back({p + "mlp.up", {ff, d}});
            t.push_back({p + "mlp.down", {d, ff}});
            t.push_back({p + "ls2", {d}});
        }
    }
    return t;
}

// a vector as one padded row
void LmBlocks::norm_row(DevBuf<bf16_t>& dst, const bf16_t* src, int n, int padded, hipStream_t s) {
    dst.alloc(padded);
    hipLaunchKernelGGL(k_place_rows, dim3(cdiv(padded, 256)), dim3(256), 0, s, src, dst.p, 1, n, 1, 0, 1, 1, 1, padded);
}
// the placed rows into a packed matrix of `total` elements, n-tile t at tile0 + t stride
void LmBlocks::pack_rows(DevBuf<bf16_t>& dst, size_t total, int Np, int Kp, int tile0, int stride, hipStream_t s) {
    if (!dst.p) { dst.alloc(total); dst.zero(s); }
    launch_pack_weight(place_.p, dst.p, Np, Kp, Np / 16, stride, tile0, s);
}
void LmBlocks::set_tensor(const std::string& name, const bf16_t* src, const std::vector<int64_t>& shape, hipStream_t s) {
    static const std::vector<int64_t> none;
    const std::vector<int64_t>* want = nullptr;
    for (int i = 0; i < L; ++i) {                                              // what belongs to the feed-forward a layer does not have scales nothing
        if (layers_[i].owner != i || layers_[i].ffp) continue;
        const std::string p = "l" + std::to_string(spec.layers[i].index) + ".";
        if (layers_[i].kind == BLOCK_LATENT ? name == p + "ls2" : name == p + "norm2" || name == p + "norm2b") return;
    }
    const auto list = tensor_list();
    for (auto& t : list) if (t.first == name) want = &t.second;
    MIS_REQUIRE(want, MIS_ERR_INVALID_INPUT, "unexpected tensor %s", name.c_str());
    MIS_REQUIRE(*want == shape, MIS_ERR_INVALID_INPUT, "%s shape mismatch", name.c_str());
    const int64_t N = shape[0], K = shape.size() > 1 ? shape[1] : 1;
    auto vec = [&](DevBuf<bf16_t>& dst, int padded) { norm_row(dst, src, (int)N, padded, s); };
    auto pack = [&](DevBuf<bf16_t>& dst, size_t total, int Np, int Kp, int tile0) { pack_rows(dst, total, Np, Kp, tile0, 1, s); };
    if (name == "embed") { place(src, N, K, 1, 0, 1, 1, V, dp, s); emb_.alloc((size_t)V * dp); HIP_CHECK(hipMemcpyAsync(emb_.p, place_.p, (size_t)V * dp * 2, hipMemcpyDeviceToDevice, s)); }
    else if (name == "embed.norm") vec(g_embed_, dp);
    else if (name == "final.norm") vec(g_final_, dp);
    else if (name == "head") { place(src, N, K, 1, 0, 1, 1, Vpad, dp, s); pack(head_, (size_t)Vpad * dp, Vpad, dp, 0); }
    else {
        const size_t dot = name.find('.');
        const int li = atoi(name.substr(1, dot - 1).c_str());
        const std::string t = name.substr(dot + 1);
        int run = 0;                                                            // the run that owns the layer's tensors
        while (layers_[run].owner != run || spec.layers[run].index != li) ++run;
        const Layer& l = layers_[run];
        if (l.kind != BLOCK_LATENT) {
            mixed_set(run, t, src, shape, s);
            HIP_CHECK(hipGetLastError());
            loaded_.insert(name);
            return;
        }
        const LatentDims& D = l.D;
        Weights& w = *w_[li];
        const int HQ = D.np + D.rp;
        const size_t w1 = (size_t)(l.Nqkv + l.ffp) * dp, ukv = (size_t)D.H * (D.np + D.vp) * D.Rp;
        if (t == "norm1") vec(w.norm1, dp);
        else if (t == "ls1") vec(w.ls1, dp);
        else if (t == "ls2") vec(w.ls2, dp);
        else if (t == "mix.dkv.norm") vec(w.c_norm, D.Rp);
        else if (t == "mix.q") { place(src, N, K, D.n, D.r, HQ, D.np, D.H * HQ, dp, s); pack(w.w1, w1, D.H * HQ, dp, 0); }
        else if (t == "mix.dkv") { place(src, N, K, D.R, D.r, D.Rp + D.rp, D.Rp, D.Rp + D.rp, dp, s); pack(w.w1, w1, D.Rp + D.rp, dp, D.H * HQ / 16); }
        else if (t == "mlp.up") { place(src, N, K, 1, 0, 1, 1, l.ffp, dp, s); pack(w.w1, w1, l.ffp, dp, l.Nqkv / 16); }
        else if (t == "mix.uk") {
            place(src, N, K, D.n, 0, D.np, D.np, D.H * D.np, D.Rp, s);
            pack(w.ukv, ukv, D.H * D.np, D.Rp, 0);
            const size_t n = (size_t)D.H * D.Rp * D.np;
            place_.alloc(n);                                                   // (stream order: the pack above has read the buffer; a larger one is a new allocation)
            hipLaunchKernelGGL(k_place_head_transposed, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, s, src, place_.p, D.H, D.n, D.R, D.Rp, D.np);
            pack(w.uk_t, n, D.H * D.Rp, D.np, 0);
        }
        else if (t == "mix.uv") { place(src, N, K, D.v, 0, D.vp, D.vp, D.H * D.vp, D.Rp, s); pack(w.ukv, ukv, D.H * D.vp, D.Rp, D.H * D.np / 16); }
        else if (t == "mix.o") { place(src, N, K, 1, 0, 1, 1, dp, l.Ko, s); pack(w.wo, (size_t)dp * l.Ko, dp, l.Ko, 0); }
        else if (t == "mlp.down") { place(src, N, K, 1, 0, 1, 1, dp, l.ffp, s); pack(w.wdown, (size_t)dp * l.ffp, dp, l.ffp, 0); }
    }
    HIP_CHECK(hipGetLastError());
    loaded_.insert(name);
}
void LmBlocks::init_synthetic(uint64_t seed, hipStream_t s) {
    uint64_t key = seed * 100000ull + 1;
    for (auto& t : tensor_list()) {
        size_t n = 1;
        for (int64_t v : t.second) n *= (size_t)v;
        stage_.alloc(n);
        const bool vec = t.second.size() == 1;
        const float amp = vec ? 0.1f : (t.first == "embed" ? 1.0f : (float)sqrt(3.0 / t.second[1]));
        launch_synth_fill_bf16(stage_.p, n, key++, amp, vec ? 1 : 0, s);
        set_tensor(t.first, stage_.p, t.second, s);
        HIP_CHECK(hipStreamSynchronize(s));
    }
    stage_.release();
}
void LmBlocks::finalize() const {
    for (auto& t : tensor_list()) MIS_REQUIRE(loaded_.count(t.first), MIS_ERR_NOT_INITIALIZED, "LM weight missing: %s", t.first.c_str());
}
double LmBlocks::weight_bytes_per_step() const {
    double b = 2.0 * V * d;
    for (int i = 0; i < L; ++i) {
        if (layers_[i].kind != BLOCK_LATENT) { b += mixed_weight_bytes(i); continue; }
        const LatentDims& D = layers_[i].D;
        b += 2.0 * ((double)D.H * (D.n + D.r) * d + (double)(D.R + D.r) * d + (double)D.H * (D.n + D.v) * D.R + (double)d * D.H * D.v + 2.0 * d * spec.layers[i].ff);
    }
    return b;
}
double LmBlocks::cache_bytes_per_key() const {
    double b = 0;
    for (auto& l : layers_) b += (l.kind == BLOCK_LATENT ? (double)(l.D.R + l.D.r) : (double)l.A.G * (l.A.D + l.A.E)) * esz();
    return b;
}

// ============================================================================ state
void LmBlocks::reset(int batch, int Smax, hipStream_t s) {
    const bool same = batch == batch_ && Smax == Smax_;
    batch_ = batch; Smax_ = Smax; Mpad_ = (int)round_up(batch, 16);
    if (Smax > rope_len_) {
        std::vector<float> cs, sn;
        for (auto& r : ropes_) {
            rotary_tables_host(r.spec, Smax, cs, sn);
            r.cs.alloc(cs.size()); r.sn.alloc(sn.size());
            if (cs.empty()) continue;
            HIP_CHECK(hipMemcpyAsync(r.cs.p, cs.data(), cs.size() * 4, hipMemcpyHostToDevice, s));
            HIP_CHECK(hipMemcpyAsync(r.sn.p, sn.data(), sn.size() * 4, hipMemcpyHostToDevice, s));
            HIP_CHECK(hipStreamSynchronize(s));
        }
        rope_len_ = Smax;
    }
    if (same) return;                                                          // (a cache row is written before it is read, a state starts with position 0)
    cache_.resize(L); state_.resize(L);
    size_t n_qkv = 0, n_act = 0, n_q = 0, n_ol = 0, n_share = 0, n_ml = 0, n_slab = 2;
    const int max_s = dp > 8192 ? 4 : 8;                                       // slabs the residual kernel takes
    for (int i = 0; i < L; ++i) {
        Layer& l = layers_[i];
        const LatentDims& D = l.D;
        if (!cache_[i]) cache_[i].reset(new DevBuf<uint8_t>());
        if (!state_[i]) state_[i].reset(new DevBuf<float>());
        if (l.kind != BLOCK_LATENT) {
            mixed_reset(i, s);
            n_qkv = std::max(n_qkv, (size_t)l.Nqkv); n_act = std::max(n_act, (size_t)l.ffp);
            n_q = std::max(n_q, (size_t)l.A.H * l.A.Dp);
            n_slab = std::max(n_slab, (size_t)std::max(l.s1, l.s2));
            n_ml = std::max(n_ml, (size_t)l.shares * batch * l.A.H * 2);
            DevBuf<uint8_t>& at = attn_[columns(i)];
            at.alloc((size_t)Mpad_ * l.Ko * esz());
            at.zero(s);
            continue;
        }
        cache_[i]->alloc((size_t)batch * Smax * D.CW * esz());
        l.shares = !f32 && latent_decode_mfma_ok(D) ? latent_decode_shares(D, batch, Smax) : 0;
        l.s1 = 1; l.s2 = l.ffp ? 1 : 0;
        if (!f32) gemm_choose_dual_split(dp / 16 / 2, l.Ko / 32, l.ffp / 32, 4, max_s, &l.s1, &l.s2);
        n_qkv = std::max(n_qkv, (size_t)l.Nqkv); n_act = std::max(n_act, (size_t)l.ffp);
        n_q = std::max(n_q, (size_t)D.H * D.CW);
        if (!l.shares) n_ol = std::max(n_ol, (size_t)D.H * D.Rp);
        n_share = std::max(n_share, (size_t)l.shares * batch * D.H * D.Rp);
        n_ml = std::max(n_ml, (size_t)l.shares * batch * D.H * 2);
        n_slab = std::max(n_slab, (size_t)(l.s1 + l.s2));
        DevBuf<uint8_t>& at = attn_[columns(i)];
        at.alloc((size_t)Mpad_ * l.Ko * esz());
        at.zero(s);
    }
    x_.alloc((size_t)Mpad_ * dp); h_.alloc((size_t)Mpad_ * dp * esz());
    qkv_.alloc((size_t)Mpad_ * n_qkv); act_.alloc((size_t)Mpad_ * std::max<size_t>(n_act, 1) * esz());
    q_.alloc((size_t)Mpad_ * n_q * esz()); olat_.alloc((size_t)Mpad_ * std::max<size_t>(n_ol, 1) * esz());
    part_.alloc(n_slab * Mpad_ * dp);
    share_.alloc(n_share); share_ml_.alloc(n_ml);
    logits_.alloc((size_t)Mpad_ * Vpad);
    mixed_buffers(mix_, Mpad_, s);
    x_.zero(s); h_.zero(s); qkv_.zero(s); act_.zero(s); q_.zero(s); olat_.zero(s); logits_.zero(s);
}

std::pair<int, int> LmBlocks::columns(int li) const {
    const Layer& l = layers_[li];
    if (l.kind == BLOCK_PARALLEL) return {l.A.H * l.A.E, l.R.W};
    return {l.kind == BLOCK_DECAY ? l.S.H * l.S.E : l.D.H * l.D.v, 0};
}
Operand LmBlocks::operand(void* p, int ld, int rows_padded, bool packed) const {
    return Operand{p, f32 ? OPK_F32 : (packed ? OPK_PACKED : OPK_ROWS), ld, std::max(1, rows_padded / 16)};
}
LatentRows LmBlocks::latent_rows(int li, const float* qkv, void* q, bool expanded, const RowTable& rows) const {
    const Layer& l = layers_[li];
    LatentRows p{};
    p.qkv = qkv; p.ld = l.Nqkv; p.c_norm = W(li).c_norm.p;
    p.rope_cos = ropes_[l.rope].cs.p; p.rope_sin = ropes_[l.rope].sn.p;
    p.rows = rows; p.cache = cache_[li]->p; p.Smax = Smax_; p.q = q;
    p.q_ld = expanded ? l.D.DK : l.D.CW; p.q_rot_off = expanded ? l.D.np : l.D.Rp; p.with_plain = expanded ? 1 : 0;
    p.f32 = f32 ? 1 : 0;
    return p;
}

// projections in qkv -> cache rows, absorbed queries, latent sums, values (operand of the output projection)
void LmBlocks::absorbed_attention(int li, const float* qkv, void* q, void* olat, const Operand& out, const RowTable& rows, int M, int shares, hipStream_t s) {
    const Layer& l = layers_[li];
    const LatentDims& D = l.D;
    const Weights& w = W(li);
    const size_t uvz = (size_t)(D.vp / 16) * (D.Rp / 32) * 512;
    const bf16_t* uv = w.ukv.p + (size_t)(D.H * D.np / 16) * (D.Rp / 32) * 512;
    const LatentRows lr = latent_rows(li, qkv, q, false, rows);
    if (f32) {
        launch_latent_rows(D, lr, M, s);
        GemmF32 g{};
        g.X = qkv; g.ldx = l.Nqkv; g.xz = D.np + D.rp; g.W = w.uk_t.p; g.wz = (size_t)(D.Rp / 16) * (D.np / 32) * 512;
        g.out = (float*)q; g.ldo = D.H * D.CW; g.oz = D.CW; g.M = M; g.NT = D.Rp / 16; g.KT = D.np / 32; g.n_valid = D.Rp; g.heads = D.H;
        launch_gemm_f32(g, s);
    } else launch_latent_absorb(D, lr, w.uk_t.p, M, s);
    LatentAttn a{};
    a.q = q; a.cache = cache_[li]->p; a.Smax = Smax_; a.rows = rows; a.out = olat; a.f32 = f32 ? 1 : 0;
    if (shares > 0) {
        LatentShares sh;
        sh.S = shares; sh.part = share_.p; sh.ml = share_ml_.p;
        launch_latent_attn_decode(D, a, sh, M, s);
        launch_latent_share_values(D, sh, uv, uvz, out, M, s);
        return;
    }
    launch_latent_attn_any(D, a, M, s);
    if (f32) {
        GemmF32 g{};
        g.X = (const float*)olat; g.ldx = D.H * D.Rp; g.xz = D.Rp; g.W = uv; g.wz = uvz;
        g.out = (float*)out.p; g.ldo = out.ld; g.oz = D.v; g.M = M; g.NT = D.vp / 16; g.KT = D.Rp / 32; g.n_valid = D.v; g.heads = D.H;
        launch_gemm_f32(g, s);
    } else launch_latent_values(D, (const bf16_t*)olat, uv, uvz, out, M, s);
}

// ============================================================================ decode step
GemmF32 gemm32(const void* X, int ldx, const bf16_t* W, float* out, int ldo, int M, int N, int K, int epi) {
    GemmF32 g{};
    g.X = (const float*)X; g.ldx = ldx; g.W = W; g.out = out; g.ldo = ldo; g.M = M; g.NT = N / 16; g.KT = K / 32; g.n_valid = N; g.epi = epi;
    return g;
}
void LmBlocks::step_layer(int li, const BlockRows& r, hipStream_t s) {
    if (layers_[li].kind != BLOCK_LATENT) { mixed_step_layer(li, r, s); return; }
    const Layer& l = layers_[li];
    const Weights& w = W(li);
    RowTable rows; rows.pos = r.pos_cur; rows.on = r.active;
    void* at = attn_[columns(li)].p;
    if (f32) {
        launch_gemm_f32(gemm32(h_.p, dp, w.w1.p, qkv_.p, l.Nqkv, batch_, l.Nqkv, dp, F32_STORE), s);
        if (l.ffp) launch_gemm_f32(gemm32(h_.p, dp, w.w1.p + (size_t)l.Nqkv * dp, (float*)act_.p, l.ffp, batch_, l.ffp, dp, F32_RELU2), s);
    } else {
        const int NT = (l.Nqkv + l.ffp) / 16;
        const bool wide = Mpad_ <= 32 && NT / 4 >= 192;                        // four n-tiles per wave where the launch still fills the chip
        GemmExtra ex; ex.out2 = act_.p; ex.split = l.Nqkv / 16;
        launch_gemm_skinny(EPI_SPLIT_RELU2, wide ? 4 : 2, wide ? 2 : 4, w.w1.p, (const bf16_t*)h_.p, qkv_.p, NT, dp / 32, 1, l.Nqkv, Mpad_, s, nullptr, wide ? 2 : 4, ex);
    }
    absorbed_attention(li, qkv_.p, q_.p, olat_.p, operand(at, l.Ko, Mpad_, true), rows, batch_, l.shares, s);
    const size_t slab = (size_t)Mpad_ * dp;
    if (f32) {
        launch_gemm_f32(gemm32(at, l.Ko, w.wo.p, part_.p, dp, batch_, dp, l.Ko, F32_STORE), s);
        if (l.ffp) launch_gemm_f32(gemm32(act_.p, l.ffp, w.wdown.p, part_.p + slab, dp, batch_, dp, l.ffp, F32_STORE), s);
    } else if (l.ffp) {
        GemmExtra ex; ex.w2 = w.wdown.p; ex.x2 = (const bf16_t*)act_.p; ex.kt2 = l.ffp / 32; ex.s1 = l.s1;
        launch_gemm_skinny(EPI_DUAL, 2, l.ffp / 32 >= 64 ? 2 : 4, w.wo.p, (const bf16_t*)at, part_.p, dp / 16, l.Ko / 32, l.s1 + l.s2, dp, Mpad_, s, nullptr, 0, ex);
    } else launch_gemm_skinny(EPI_PARTIAL, 2, 4, w.wo.p, (const bf16_t*)at, part_.p, dp / 16, l.Ko / 32, l.s1, dp, Mpad_, s);
    const ScaledSlabs sl{part_.p, l.s1, l.s2, w.ls1.p, w.ls2.p};
    launch_scaled_residual_norm(sl, Mpad_, x_.p, norm_after(li), operand(h_.p, dp, Mpad_, true), d, dp, spec.eps, f32 ? batch_ : Mpad_, s);
}
void LmBlocks::enqueue_step(const BlockRows& r, hipStream_t s) {
    launch_rows_embed_norm2(emb_.p, r.ids, V, g_embed_.p, W(0).norm1.p, x_.p, operand(h_.p, dp, Mpad_, true), d, dp, spec.eps, batch_, Mpad_, r.active, r.pos_cur,
                            r.pos_next, s, spec.norm_add);
    for (int li = 0; li < L; ++li) step_layer(li, r, s);
}
// operand rows -> float32 logits [rows][Vpad]
void LmBlocks::head_rows(const void* op, bool packed, int rows, int rows_padded, float* out, hipStream_t s) {
    if (f32) {
        GemmF32 g = gemm32(op, dp, head_.p, out, Vpad, rows, Vpad, dp, F32_SOFTCAP);
        g.scale = spec.logit_scale; g.cap = spec.softcap;
        launch_gemm_f32(g, s);
    } else if (packed) {
        GemmExtra ex; ex.scale = spec.logit_scale; ex.cap = spec.softcap;
        const bool wide = rows_padded <= 32 && Vpad / 64 >= 192;
        launch_gemm_skinny(EPI_SOFTCAP, wide ? 4 : 2, 4, head_.p, (const bf16_t*)op, out, Vpad / 16, dp / 32, 1, Vpad, rows_padded, s, nullptr, 0, ex);
    } else {
        PfExtra ex; ex.ldc = Vpad; ex.scale = spec.logit_scale; ex.cap = spec.softcap;
        launch_gemm_pf(PF_SOFTCAP, (const bf16_t*)op, head_.p, out, rows, Vpad, dp, s, ex);
    }
}
void LmBlocks::enqueue_head(hipStream_t s) { head_rows(h_.p, true, batch_, Mpad_, logits_.p, s); }

// ============================================================================ prompt pass
void LmBlocks::pass_layer(int li, int M, const RowTable& rows, int n_tiles, int Mk, hipStream_t s) {
    const Layer& l = layers_[li];
    const LatentDims& D = l.D;
    const Weights& w = W(li);
    void* at = pattn_[columns(li)].p;
    if (f32) {
        launch_gemm_f32(gemm32(ph_.p, dp, w.w1.p, pqkv_.p, l.Nqkv, M, l.Nqkv, dp, F32_STORE), s);
        if (l.ffp) launch_gemm_f32(gemm32(ph_.p, dp, w.w1.p + (size_t)l.Nqkv * dp, (float*)pact_.p, l.ffp, M, l.ffp, dp, F32_RELU2), s);
    } else {
        PfExtra ex; ex.ldc = l.Nqkv; ex.split = l.Nqkv / 16; ex.out2 = pact_.p; ex.ld2 = l.ffp;
        launch_gemm_pf(PF_SPLIT_RELU2, (const bf16_t*)ph_.p, w.w1.p, pqkv_.p, M, l.Nqkv + l.ffp, dp, s, ex);
    }
    if (n_tiles > 0 && latent_prefill_mfma_ok(D)) {
        launch_latent_rows(D, latent_rows(li, pqkv_.p, pq_.p, true, rows), M, s);
        const int Nkv = D.H * (D.np + D.vp);
        PfExtra ex; ex.ldx = D.CW; ex.xrow = pkey_.p; ex.ldc = Nkv;
        launch_gemm_pf(PF_ROWS_BF16, (const bf16_t*)cache_[li]->p, w.ukv.p, pkv_.p, Mk, Nkv, D.Rp, s, ex);
        LatentPrefill a{};
        a.q = (const bf16_t*)pq_.p; a.kv = pkv_.p; a.ldkv = Nkv; a.cache = (const bf16_t*)cache_[li]->p; a.Smax = Smax_; a.tiles = ptiles_.p; a.n_tiles = n_tiles;
        a.out = (bf16_t*)at; a.ldo = l.Ko;
        launch_latent_attn_prefill(D, a, s);
    } else absorbed_attention(li, pqkv_.p, pq_.p, polat_.p, operand(at, l.Ko, 0, false), rows, M, 0, s);
    if (f32) {
        GemmF32 g = gemm32(at, l.Ko, w.wo.p, px_.p, dp, M, dp, l.Ko, F32_ADD_SCALED);
        g.ls = w.ls1.p;
        launch_gemm_f32(g, s);
        if (l.ffp) { g = gemm32(pact_.p, l.ffp, w.wdown.p, px_.p, dp, M, dp, l.ffp, F32_ADD_SCALED); g.ls = w.ls2.p; launch_gemm_f32(g, s); }
    } else {
        PfExtra ex; ex.ldc = dp; ex.ls = w.ls1.p;
        launch_gemm_pf(PF_SCALED_ADD, (const bf16_t*)at, w.wo.p, px_.p, M, dp, l.Ko, s, ex);
        ex.ls = w.ls2.p;
        if (l.ffp) launch_gemm_pf(PF_SCALED_ADD, (const bf16_t*)pact_.p, w.wdown.p, px_.p, M, dp, l.ffp, s, ex);
    }
    if (li + 1 < L) launch_gather_norm(px_.p, nullptr, norm_after(li), operand(ph_.p, dp, 0, false), d, dp, spec.eps, M, s);
}

void LmBlocks::pass(const std::vector<PassEntry>& entries, const std::vector<int32_t>& tokens, const std::vector<int32_t>& want, float* logits_out,
                    float* residual_out, bool last_rows, hipStream_t s) {
    const size_t total = tokens.size();
    // the layers of one model may differ in window and sizes: key rows and buffers are laid out for the widest
    int max_window = 0;
    bool all_keys = false, expanded = !f32;
    size_t n_qkv = 0, n_act = 1, n_q = 0, n_ol = 1, n_kv = 0;
    bool latent = false;
    for (auto& l : layers_) {
        n_qkv = std::max(n_qkv, (size_t)l.Nqkv); n_act = std::max(n_act, (size_t)l.ffp);
        if (l.kind != BLOCK_LATENT) { n_q = std::max(n_q, (size_t)l.A.H * l.A.Dp); continue; }
        latent = true;
        const bool ex = !f32 && latent_prefill_mfma_ok(l.D);
        expanded = expanded && ex;
        all_keys = all_keys || l.D.window <= 0;
        max_window = std::max(max_window, l.D.window);
        n_q = std::max(n_q, (size_t)l.D.H * std::max(l.D.CW, l.D.DK)); n_ol = std::max(n_ol, (size_t)l.D.H * l.D.Rp);
        n_kv = std::max(n_kv, (size_t)l.D.H * (l.D.np + l.D.vp));
    }
    const size_t cap = std::min<size_t>(total, std::max(1, pass_rows));
    px_.alloc(cap * dp); ph_.alloc(cap * dp * esz()); pqkv_.alloc(cap * n_qkv); pact_.alloc(cap * n_act * esz());
    pq_.alloc(cap * n_q * esz());
    if (latent && !expanded) polat_.alloc(cap * n_ol * esz());
    mixed_buffers(pmix_, (int)cap, s);
    for (int i = 0; i < L; ++i) {
        DevBuf<uint8_t>& at = pattn_[columns(i)];
        const size_t bytes = cap * layers_[i].Ko * esz();
        if (at.n < bytes) { at.alloc(bytes); at.zero(s); }                     // K padding columns: zero from here on
    }
    pids_.alloc(cap); pseq_.alloc(cap); ppos_.alloc(cap); ppos0_.alloc(cap);
    size_t ei = 0, done_in_entry = 0, t0 = 0;
    while (t0 < total) {
        const size_t n = std::min(cap, total - t0);
        std::vector<int32_t> seq(n), pos(n), pos0(n), keys;
        std::vector<LatentTile> tiles;
        std::vector<RowSpan> spans, qtiles;
        std::vector<RecurChunk> chunks;
        std::vector<std::pair<int32_t, int32_t>> last;                         // (row, sequence) of entries that end in this chunk
        size_t at = 0;
        while (at < n) {
            const PassEntry& e = entries[ei];
            const size_t take = std::min(n - at, (size_t)e.n - done_in_entry);
            const int p0 = e.pos0 + (int)done_in_entry;
            for (size_t k = 0; k < take; ++k) { seq[at + k] = e.seq; pos[at + k] = p0 + (int)k; pos0[at + k] = p0; }
            spans.push_back(RowSpan{(int)at, (int)take, e.seq, p0});
            for (size_t q = 0; q < take; q += RECUR_CHUNK)
                chunks.push_back(RecurChunk{RowSpan{(int)(at + q), (int)std::min<size_t>(RECUR_CHUNK, take - q), e.seq, p0 + (int)q}, (int)spans.size() - 1, p0,
                                            (int)(q / RECUR_CHUNK), q + RECUR_CHUNK >= take ? 1 : 0});
            for (size_t q = 0; q < take; q += GROUPED_QT)
                qtiles.push_back(RowSpan{(int)(at + q), (int)std::min<size_t>(GROUPED_QT, take - q), e.seq, p0 + (int)q});
            if (!f32 && latent) {
                const int kp0 = all_keys ? 0 : std::max(0, p0 - max_window + 1), krow0 = (int)keys.size();
                for (int p = kp0; p < p0 + (int)take; ++p) keys.push_back(e.seq * Smax_ + p);
                for (size_t q = 0; q < take; q += LATENT_QT)
                    tiles.push_back(LatentTile{(int)(at + q), (int)std::min<size_t>(LATENT_QT, take - q), e.seq, p0 + (int)q, krow0, kp0});
            }
            at += take; done_in_entry += take;
            if (done_in_entry == (size_t)e.n) { last.push_back({(int)at - 1, e.seq}); ++ei; done_in_entry = 0; }
        }
        std::vector<DecaySegment> segs;
        if (const Layer* big = widest_decay()) {
            const int len = decay_segment_rows(big->S, (int)n, (int)spans.size());
            for (auto& sp : spans)
                for (int at2 = 0, k = 0, count = cdiv(sp.n, len); at2 < sp.n; at2 += len, ++k)
                    segs.push_back(DecaySegment{RowSpan{sp.row0 + at2, std::min(len, sp.n - at2), sp.seq, sp.pos0 + at2}, k, count, len, sp.pos0});
            psegs_.alloc(segs.size());
            HIP_CHECK(hipMemcpyAsync(psegs_.p, segs.data(), segs.size() * sizeof(DecaySegment), hipMemcpyHostToDevice, s));
            if (!f32 && segs.size() > spans.size()) pmix_.ends.alloc(segs.size() * big->S.H * big->S.D * big->S.Es);
        }
        HIP_CHECK(hipMemcpyAsync(pids_.p, tokens.data() + t0, n * 4, hipMemcpyHostToDevice, s));
        HIP_CHECK(hipMemcpyAsync(pseq_.p, seq.data(), n * 4, hipMemcpyHostToDevice, s));
        HIP_CHECK(hipMemcpyAsync(ppos_.p, pos.data(), n * 4, hipMemcpyHostToDevice, s));
        HIP_CHECK(hipMemcpyAsync(ppos0_.p, pos0.data(), n * 4, hipMemcpyHostToDevice, s));
        pspans_.alloc(spans.size());
        HIP_CHECK(hipMemcpyAsync(pspans_.p, spans.data(), spans.size() * sizeof(RowSpan), hipMemcpyHostToDevice, s));
        pqtiles_.alloc(qtiles.size());
        HIP_CHECK(hipMemcpyAsync(pqtiles_.p, qtiles.data(), qtiles.size() * sizeof(RowSpan), hipMemcpyHostToDevice, s));
        pchunks_.alloc(chunks.size());
        HIP_CHECK(hipMemcpyAsync(pchunks_.p, chunks.data(), chunks.size() * sizeof(RecurChunk), hipMemcpyHostToDevice, s));
        if (!f32 && latent) {
            pkey_.alloc(keys.size()); ptiles_.alloc(tiles.size());
            pkv_.alloc(keys.size() * n_kv);
            HIP_CHECK(hipMemcpyAsync(pkey_.p, keys.data(), keys.size() * 4, hipMemcpyHostToDevice, s));
            HIP_CHECK(hipMemcpyAsync(ptiles_.p, tiles.data(), tiles.size() * sizeof(LatentTile), hipMemcpyHostToDevice, s));
        }
        RowTable rows; rows.seq = pseq_.p; rows.pos = ppos_.p;
        MixRows mr;
        mr.rows = rows; mr.pos0 = ppos0_.p; mr.spans.span = pspans_.p; mr.M = (int)n; mr.n_spans = (int)spans.size(); mr.tiles = pqtiles_.p; mr.n_tiles = (int)qtiles.size();
        mr.chunks = pchunks_.p; mr.n_chunks = (int)chunks.size(); mr.segs = psegs_.p; mr.n_segs = (int)segs.size();
        launch_rows_embed_norm2(emb_.p, pids_.p, V, g_embed_.p, W(0).norm1.p, px_.p, operand(ph_.p, dp, 0, false), d, dp, spec.eps, (int)n, (int)n, nullptr, nullptr,
                                nullptr, s, spec.norm_add);
        for (int li = 0; li < L; ++li) {
            if (layers_[li].kind != BLOCK_LATENT) mixed_pass_layer(li, mr, s);
            else pass_layer(li, (int)n, rows, (int)tiles.size(), (int)keys.size(), s);
            if (residual_out)
                HIP_CHECK(hipMemcpy2DAsync(residual_out + ((size_t)li * total + t0) * d, (size_t)d * 4, px_.p, (size_t)dp * 4, (size_t)d * 4, n, hipMemcpyDeviceToHost, s));
        }
        // wanted places of this chunk, in the caller's order: up to 64 rows through the step's head GEMM, more as row-major tiles
        std::vector<int32_t> wr, wo;
        for (size_t k = 0; k < want.size(); ++k)
            if (want[k] >= (int64_t)t0 && want[k] < (int64_t)(t0 + n)) { wr.push_back(want[k] - (int)t0); wo.push_back((int)k); }
        const size_t slice = wr.size() <= 64 ? 64 : 512;
        for (size_t k = 0; k < wr.size(); k += slice) {
            const int m = (int)std::min(slice, wr.size() - k), mp = (int)round_up(m, 16);
            const bool packed = slice == 64;
            pwant_.alloc(512); phead_.alloc((size_t)slice * dp * esz()); plog_.alloc((size_t)slice * Vpad);
            HIP_CHECK(hipMemcpyAsync(pwant_.p, wr.data() + k, m * 4, hipMemcpyHostToDevice, s));
            if (packed) phead_.zero(s);
            launch_gather_norm(px_.p, pwant_.p, g_final_.p, operand(phead_.p, dp, mp, packed), d, dp, spec.eps, m, s, spec.norm_add);
            head_rows(phead_.p, packed, m, mp, plog_.p, s);
            for (int j = 0; j < m; ++j)
                HIP_CHECK(hipMemcpyAsync(logits_out + (size_t)wo[k + j] * V, plog_.p + (size_t)j * Vpad, (size_t)V * 4, hipMemcpyDeviceToHost, s));
            HIP_CHECK(hipStreamSynchronize(s));
        }
        if (last_rows)                                                         // the stream of a request's last token becomes its batch row's
            for (auto& q : last)
                HIP_CHECK(hipMemcpyAsync(x_.p + (size_t)q.second * dp, px_.p + (size_t)q.first * dp, (size_t)dp * 4, hipMemcpyDeviceToDevice, s));
        HIP_CHECK(hipStreamSynchronize(s));                                    // (the host tables above are reused by the next chunk)
        t0 += n;
    }
    if (last_rows) launch_gather_norm(x_.p, nullptr, g_final_.p, operand(h_.p, dp, Mpad_, true), d, dp, spec.eps, f32 ? batch_ : Mpad_, s, spec.norm_add);
    HIP_CHECK(hipGetLastError());
}

__global__ void k_operand_rows_f32(Operand h, float* __restrict__ out, int d, int rows) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= (size_t)rows * d) return;
    const int m = (int)(i / d), k = (int)(i - (size_t)m * d);
    out[i] = h.kind == OPK_F32 ? ((const float*)h.p)[(size_t)m * h.ld + k] : bf16_to_f32(((const bf16_t*)h.p)[xpk_index(m, k, h.MT)]);
}
void LmBlocks::final_norm_rows(float* out, int rows, hipStream_t s) {
    plog_.alloc((size_t)rows * d);
    hipLaunchKernelGGL(k_operand_rows_f32, dim3((unsigned)(((size_t)rows * d + 255) / 256)), dim3(256), 0, s, operand(h_.p, dp, Mpad_, true), plog_.p, d, rows);
    HIP_CHECK(hipMemcpyAsync(out, plog_.p, (size_t)rows * d * 4, hipMemcpyDefault, s));
    HIP_CHECK(hipStreamSynchronize(s));
}
