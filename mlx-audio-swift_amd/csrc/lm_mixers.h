// lm_mixers.h - token mixers of layer-list language models (lm_blocks.hip) beside latent attention: grouped attention under a sliding window with
// kept first tokens and a sink, the gated linear recurrence behind a short convolution, attention with a decayed outer-product state; and the
// residual step of a layer that norms a sublayer's result before it is added.  Every size and constant is a parameter.
#pragma once
#include "common.h"
#include "lm_latent.h"

// Rows of a pass by request: rows row0 .. row0 + n - 1 are positions pos0 .. of sequence seq.  span null: a decode step - row i is sequence i at
// position pos[i], rows with on[i] = 0 do nothing (on null: all).  A sequence's state counts from its position 0: what a slot held before is
// not looked at.
struct RowSpan { int32_t row0, n, seq, pos0; };
struct SpanTable { const RowSpan* span = nullptr; const int32_t* pos = nullptr; const uint8_t* on = nullptr; };

// ---- residual step: y = (sum of S slabs [S][slab_rows][dp]) * r + bias * bias_scale;  x += rms(y) * (g_post + g_add);  operand = rms(x) * (g_next + g_add).
// r: ss null: 1; otherwise 1 / sqrt(sum(ss[m][0 .. n_ss)) / ss_cols + eps) - a norm of the product's input that waited until behind the product
struct SublayerOut { const float* p = nullptr; int S = 1; const float* ss = nullptr; int n_ss = 0, ss_cols = 1; const bf16_t* bias = nullptr; float bias_scale = 1.0f; };
void launch_post_norm_residual(const SublayerOut& y, int slab_rows, float* x, const bf16_t* g_post, const bf16_t* g_next, float g_add, const Operand& h, int d, int dp,
                               float eps, int rows, hipStream_t s);
// act[m][j] = silu(g) * u on float32 rows of interleaved 16-column tiles (gate, up, gate, ...)
void launch_swiglu_rows_f32(const float* gu, int ldg, float* act, int lda, int ffp, int rows, hipStream_t s);

// ---- grouped attention
struct GroupedDims {
    int H, G, D, E;             // query heads, key / value heads, query-key size, value size
    int Dp, Ep;                 // padded: D % 32, E % 16
    int window, keep;           // keys a position sees, itself included (0: all), and the first tokens it sees whatever the distance
    int rot;                    // rotated dimensions; pair (i, i + rot / 2)
    float scale, eps;
};
GroupedDims grouped_dims(int H, int G, int D, int E, int window, int keep, int rot, float scale, float eps);
// Caches, bf16: matrix-core fragments.  keys [seq][G][Smax / 16][Dp / 32][64][8]: lane q * 16 + i holds dims 8 q .. + 7 of key i; values
// [seq][G][Smax / 32][Ep / 16][64][8]: lane q * 16 + i holds value column i of keys 4 q .. + 3 and 16 + 4 q .. + 3, the order in which a pair of
// score tiles leaves the weights in a lane.  float32: rows [seq][G][Smax][Dp], [seq][G][Smax][Ep].
struct GroupedRows {            // projections of a pass (without their biases) -> cache and query rows
    const float* proj; int ld, oq, ok, ov;
    const bf16_t* bias;         // [ld]
    const bf16_t *qn, *kn;      // [D]
    const float *rope_cos, *rope_sin;      // [positions][rot / 2]
    RowTable rows;
    void *kc, *vc; int Smax;
    void* q;                    // [rows][H][Dp]
    int f32;
};
void launch_grouped_rows(const GroupedDims& D, const GroupedRows& p, int rows, hipStream_t s);
struct GroupedAttn {
    const void* q; const void *kc, *vc; int Smax;
    const bf16_t* sink;         // [H]
    RowTable rows;
    Operand out; float out_scale;           // head a at columns a E ..
    int f32;
};
// any sizes, either element type; the cache holds the rows already
void launch_grouped_attn_any(const GroupedDims& D, const GroupedAttn& p, int rows, hipStream_t s);
// matrix cores, bf16 (lm_grouped.hip)
bool grouped_mfma_ok(const GroupedDims& D);
#define GROUPED_QT 64           // queries of one request per prompt tile
// launch_grouped_rows for the rows of a prompt pass (bf16)
void launch_grouped_rows_prefill(const GroupedDims& D, const GroupedRows& p, const RowSpan* tiles, int n_tiles, int rows, hipStream_t s);
void launch_grouped_attn_prefill(const GroupedDims& D, const GroupedAttn& p, const RowSpan* tiles, int n_tiles, hipStream_t s);
// ---- gated linear recurrence: u = conv(x);  r, g = sigmoid(block-diagonal products of u);  S = a S + sqrt(1 - a^2) g u, a = exp(-c r)
struct RecurDims {
    int W, B, n, taps;          // channels, blocks, channels per block, convolution taps
    int np, nt;                 // block size padded to 32 (columns of the products), 16-row tiles of a block
};
RecurDims recur_dims(int W, int B, int taps);
struct RecurParams {
    const float* proj; int ld, oy, ox;
    const bf16_t* bias;         // [ld]
    const bf16_t *conv, *conv_b, *ra_b, *ri_b;
    const bf16_t *ra, *ri;      // packed per block [B][nt][np / 32][64][8]
    const float *conv_t, *conv_b32, *bias_x;        // [taps][W], [W], [W]: the same values in float32, channels side by side
    const float* c;             // [W] 8 softplus(lam)
    RowTable rows; const int32_t* pos0;     // pos0: first position of the row's span (null: the row's own)
    SpanTable spans;
    float* state;               // [seq][W]
    float* hist;                // [seq][taps][W]: the convolution's input at position p in slot p % taps
    Operand out; int col0; float out_scale;
};
// u [rows][B][np] float32 (columns n .. np zero)
void launch_conv_rows(const RecurDims& D, const RecurParams& p, float* u, int rows, hipStream_t s);
// raw products [rows][B][nt 16] -> recurrence along every span, times gelu of the other branch; leaves state and history behind the span
void launch_gated_scan_any(const RecurDims& D, const RecurParams& p, const float* u, const float* raw_r, const float* raw_g, int spans, hipStream_t s);
// matrix cores, bf16 (lm_recurrent.hip).  Decode: convolution, gates, state, operand in one launch
void launch_recur_step(const RecurDims& D, const RecurParams& p, int rows, hipStream_t s);
// prompt: spans in chunks of RECUR_CHUNK rows (only the last of a span may be shorter)
#define RECUR_CHUNK 64
struct RecurChunk { RowSpan rows; int32_t span, span_pos0, index, last; };      // index: in the span; last: of the span
void launch_recur_prefill(const RecurDims& D, const RecurParams& p, const RecurChunk* chunks, int n_chunks, float* loc, float* dec, float* carry0, hipStream_t s);
// float32 copies [taps][W], [W], [W] of the convolution's weights and bias and of the input's bias
void launch_conv_tables(const bf16_t* conv, const bf16_t* conv_b, const bf16_t* bias_x, float* conv_t, float* conv_b32, float* bias_x32, int W, int taps, hipStream_t s);
void launch_softplus_scaled(const bf16_t* lam, float* out, int n, float scale, hipStream_t s);

// ---- grouped attention, decode: queries, cache rows, attention and (more than one share) the shares' sum; p.q is not used.  RD, rp non-null: a gated
// recurrence on the same projections advances in the same launch
struct GroupedShares { int S = 1; float *part = nullptr, *ml = nullptr; };      // part [S][rows][H][Ep], ml [S][rows][H][2]
int grouped_decode_shares(const GroupedDims& D, int rows, int Smax);
void launch_grouped_attn_decode(const GroupedDims& D, const GroupedRows& r, const GroupedAttn& p, const GroupedShares& sh, const RecurDims* RD, const RecurParams* rp, int rows,
                                hipStream_t s);

// ---- attention with a decayed outer-product state, per head: S = c S + k v^T, o = S^T q
struct DecayDims { int H, D, E, Es, ns; };              // Es: row stride of the state (E % 64), ns: column slices of 64
DecayDims decay_dims(int H, int D, int E);
struct DecayParams {
    const float* proj; int ld, oq, ok, ov, og;          // raw projections; q, k, v go through silu, the gate through a sigmoid
    const bf16_t* act;          // prompt on the matrix cores, instead of proj: silu(q, k, v), sigmoid(gate)
    const float* decay;         // [H]
    const bf16_t* norm;         // [H E]
    SpanTable spans;
    float* state;               // [seq][H][D][Es]
    Operand out;                // o * norm * sigmoid(gate), not yet divided by the row's root mean square
    float* ss;                  // [rows][H ns] sums of squares of o
};
// any sizes, either element type
void launch_decay_any(const DecayDims& D, const DecayParams& p, int spans, hipStream_t s);
// bf16 (lm_recurrent.hip)
bool decay_mfma_ok(const DecayDims& D);
void launch_decay_step(const DecayDims& D, const DecayParams& p, int rows, hipStream_t s);
// segment index of count of one request's rows in this pass, all but the last `length` rows long (a multiple of 64); a request's segments follow each
// other in the table.  cut: some request has more than one; ends: [n_segs][H][D][Es]
struct DecaySegment { RowSpan rows; int32_t index, count, length, span_pos0; };
int decay_segment_rows(const DecayDims& D, int rows, int spans);       // length to cut `rows` rows of `spans` requests into
void launch_decay_prefill(const DecayDims& D, const DecayParams& p, const DecaySegment* segs, int n_segs, bool cut, float* ends, hipStream_t s);
