// lm_blocks.h - language models described layer by layer (config.json "layers"): weights, caches, the decode step and the prompt pass.  The
// engine around it - handles, batch rows, positions, sampler, generate loop, captured graphs - is lm_engine.hip's.
#pragma once
#include <deque>
#include <map>
#include <memory>
#include <set>
#include "lm_latent.h"
#include "lm_mixers.h"

// ---- configuration
struct LatentMixerSpec { int heads = 0, dim = 0, rot_dim = 0, vdim = 0, kv_rank = 0, window = 0; float scale = 1.0f; RotarySpec rot; };
struct GroupedMixerSpec { int heads = 0, kv_heads = 0, dim = 0, vdim = 0, window = 0, keep = 0; float scale = 1.0f; RotarySpec rot; };
struct RecurMixerSpec { int width = 0, blocks = 0, conv = 0; };
struct DecayMixerSpec { int heads = 0, dim = 0, vdim = 0; std::vector<float> decay; };
// BLOCK_LATENT: one norm, mixer and feed-forward side by side, each with a layer scale.  The others: mixer, then feed-forward, each with a norm
// before it and one behind it; BLOCK_DECAY mixes with `decay`, BLOCK_PARALLEL with left_scale * `grouped` + right_scale * `recur`.
enum { BLOCK_LATENT = 0, BLOCK_DECAY = 1, BLOCK_PARALLEL = 2 };
struct BlockSpec {
    int kind = BLOCK_LATENT;
    LatentMixerSpec mix; GroupedMixerSpec grouped; RecurMixerSpec recur; DecayMixerSpec decay;
    float left_scale = 1.0f, right_scale = 1.0f;
    int ff = 0 /* 0: no feed-forward */;
    int weights_of = -1;        // run whose weights this one uses (-1: its own)
    int index = 0;              // place in config.json's list: the tensors' prefix
};
struct BlockModelSpec {
    std::string architecture;
    int width = 0, vocab = 0;
    float eps = 1e-6f, logit_scale = 1.0f, softcap = 0.0f;
    bool embed_norm = true;     // the embedding goes through a norm of its own
    float norm_add = 0.0f;      // added to the weights of the norms over the width
    std::vector<BlockSpec> layers;      // in the order they run; a layer that runs again is listed again, with its own cache or state
};
// architectures this engine serves, by config.json "architecture"
bool block_architecture_known(const std::string& name);
BlockModelSpec parse_block_model(const JsonValue& cfg);

// ---- one request's share of a prompt pass
struct PassEntry { int seq, pos0, n; };

// Device state of the batch rows, owned by the engine
struct BlockRows { const int32_t* ids; const uint8_t* active; int32_t *pos_cur, *pos_next; };

int pad_k(int k);                // K of a GEMM operand
GemmF32 gemm32(const void* X, int ldx, const bf16_t* W, float* out, int ldo, int M, int N, int K, int epi);

class LmBlocks {
public:
    LmBlocks(const BlockModelSpec& spec, bool f32);
    const BlockModelSpec spec;
    const bool f32;                     // 32-bit mode: float32 operands, caches and GEMMs (weights stay bf16, exact in float32)
    int d, dp, V, Vpad, L;

    // weights: `src` bf16 row-major on the device; throws on an unknown name or a wrong shape
    void set_tensor(const std::string& name, const bf16_t* src, const std::vector<int64_t>& shape, hipStream_t s);
    std::vector<std::pair<std::string, std::vector<int64_t>>> tensor_list() const;      // every tensor the configuration implies
    void init_synthetic(uint64_t seed, hipStream_t s);
    void finalize() const;              // throws when a tensor is missing

    // caches and step buffers for `batch` rows of up to Smax positions
    void reset(int batch, int Smax, hipStream_t s);
    // one token of every active row (captured in the engine's decode graph); leaves the final norm of every row as the head's operand
    void enqueue_step(const BlockRows& r, hipStream_t s);
    void enqueue_head(hipStream_t s);   // logits of the batch rows: float32 [Mpad][Vpad]
    float* logits() { return logits_.p; }
    // tokens of several requests at their positions, in chunks of at most pass_rows rows.  want: places in `tokens` whose logits go to
    // logits_out [n_want][V] (host); residual_out (host, nullable): [L][tokens][d].  last_rows: leave the final norm of every entry's
    // last token as operand row `seq` of the head (what enqueue_step leaves).
    void pass(const std::vector<PassEntry>& entries, const std::vector<int32_t>& tokens, const std::vector<int32_t>& want, float* logits_out,
              float* residual_out, bool last_rows, hipStream_t s);
    void final_norm_rows(float* out, int rows, hipStream_t s);     // the head's operand as float32 [rows][d] (host or device)
    int pass_rows = 4096;
    double weight_bytes_per_step() const, cache_bytes_per_key() const;

private:
    struct Weights {                    // one set per layer that owns tensors
        DevBuf<bf16_t> w1;              // packed [(Nqkv + ffp) / 16][dp / 32]: q | latent | rotary key | up
        DevBuf<bf16_t> c_norm, norm1, ls1, ls2;
        DevBuf<bf16_t> uk_t;            // packed per head [Rp / 16][np / 32]  (absorbed form)
        DevBuf<bf16_t> ukv;             // packed [(H np + H vp) / 16][Rp / 32] (expanded form; its value part serves the absorbed form too)
        DevBuf<bf16_t> wo, wdown;       // packed [dp / 16][Ko / 32], [dp / 16][ffp / 32]
        // BLOCK_DECAY, BLOCK_PARALLEL (lm_blocks_mixed.hip).  w1 holds the mixer's input projections alone, wo both sides' output projections along K
        DevBuf<bf16_t> norm1b, norm2, norm2b, wgu /* gate and up tiles in turn */, bias1, bias_o, wo_rows, mix_norm, qn, kn, sink, conv, conv_b, ra, ri, ra_b, ri_b;
        DevBuf<float> decay, recur_c, conv32 /* launch_conv_tables */;
    };
    struct Layer {
        LatentDims D; int owner, ffp, Nqkv, Ko, shares = 1, s1 = 1, s2 = 0, rope = 0;
        int kind = BLOCK_LATENT, KR = 0 /* first operand column of the right side */;
        int oq = 0, ok = 0, ov = 0, og = 0, oy = 0, ox = 0;      // columns of the input projections
        GroupedDims A; RecurDims R; DecayDims S;
    };
    std::vector<Layer> layers_;
    std::vector<std::unique_ptr<Weights>> w_;
    std::set<std::string> loaded_;
    std::set<int> x_bias_set_;          // layers whose recurrence has its input bias
    DevBuf<bf16_t> emb_, g_embed_, g_final_, head_;
    struct Rope { RotarySpec spec; DevBuf<float> cs, sn; };
    std::deque<Rope> ropes_;
    DevBuf<bf16_t> stage_, place_;

    int batch_ = 0, Mpad_ = 0, Smax_ = 0, rope_len_ = 0;
    std::vector<std::unique_ptr<DevBuf<uint8_t>>> cache_;
    std::vector<std::unique_ptr<DevBuf<float>>> state_;          // recurrent state (and convolution history) of a layer run
    // step buffers; bf16 ones hold float32 in the 32-bit mode (sized in bytes)
    DevBuf<float> x_, qkv_, part_, share_ml_, logits_;
    DevBuf<bf16_t> share_;
    DevBuf<uint8_t> h_, act_, q_, olat_;
    std::map<std::pair<int, int>, DevBuf<uint8_t>> attn_;        // per columns in use: those between and up to the K padding stay zero
    // pass buffers
    DevBuf<float> px_, pqkv_, plog_;
    DevBuf<uint8_t> ph_, pact_, pq_, polat_, phead_;
    DevBuf<bf16_t> pkv_;
    std::map<std::pair<int, int>, DevBuf<uint8_t>> pattn_;
    DevBuf<int32_t> pids_, pseq_, ppos_, ppos0_, pkey_, pwant_;
    DevBuf<LatentTile> ptiles_;
    DevBuf<RowSpan> pspans_, pqtiles_;
    DevBuf<RecurChunk> pchunks_;
    DevBuf<DecaySegment> psegs_;
    // what the mixers of a step / a pass leave behind each other
    struct MixBuffers { DevBuf<float> u, raw_r, raw_g, ss, gu, part, ends; } mix_, pmix_;
    // rows of one pass as the mixers see them
    struct MixRows { RowTable rows; const int32_t* pos0; SpanTable spans; int M, n_spans; const RowSpan* tiles = nullptr; int n_tiles = 0; const RecurChunk* chunks = nullptr; int n_chunks = 0; const DecaySegment* segs = nullptr; int n_segs = 0; };

    int esz() const { return f32 ? 4 : 2; }
    const Weights& W(int li) const { return *w_[layers_[li].owner]; }
    void place(const bf16_t* src, int64_t N, int64_t K, int part1, int part2, int g_out, int off2, int Np, int Kp, hipStream_t s);
    Operand operand(void* p, int ld, int rows_padded, bool packed) const;
    LatentRows latent_rows(int li, const float* qkv, void* q, bool expanded, const RowTable& rows) const;
    std::pair<int, int> columns(int li) const;
    const Layer* widest_decay() const {              // the layer with the largest decayed state (null: none)
        const Layer* w = nullptr;
        for (auto& l : layers_)
            if (l.kind == BLOCK_DECAY && (!w || (size_t)l.S.H * l.S.D * l.S.Es > (size_t)w->S.H * w->S.D * w->S.Es)) w = &l;
        return w;
    }
    void norm_row(DevBuf<bf16_t>& dst, const bf16_t* src, int n, int padded, hipStream_t s);
    void pack_rows(DevBuf<bf16_t>& dst, size_t total, int Np, int Kp, int tile0, int stride, hipStream_t s);
    // BLOCK_DECAY, BLOCK_PARALLEL
    void mixed_layer(int li);
    void mixed_tensors(int li, std::vector<std::pair<std::string, std::vector<int64_t>>>& t) const;
    void mixed_set(int li, const std::string& t, const bf16_t* src, const std::vector<int64_t>& shape, hipStream_t s);
    double mixed_weight_bytes(int li) const;
    void mixed_reset(int li, hipStream_t s);
    void mixed_buffers(MixBuffers& b, int rows, hipStream_t s);
    void mixer(int li, const float* proj, void* q, const Operand& out, const MixRows& r, MixBuffers& b, hipStream_t s);
    void mixed_step_layer(int li, const BlockRows& r, hipStream_t s);
    void mixed_pass_layer(int li, const MixRows& r, hipStream_t s);
    const bf16_t* norm_after(int li) const { return li + 1 < L ? W(li + 1).norm1.p : g_final_.p; }
    void step_layer(int li, const BlockRows& r, hipStream_t s);
    void pass_layer(int li, int M, const RowTable& rows, int n_tiles, int Mk, hipStream_t s);
    // shares > 0 (decode, bf16): the keys of a row in that many shares on the matrix cores; 0: the kernels for any sizes
    void absorbed_attention(int li, const float* qkv, void* q, void* olat, const Operand& out, const RowTable& rows, int M, int shares, hipStream_t s);
    void head_rows(const void* operand, bool packed, int rows, int rows_padded, float* out, hipStream_t s);
};
