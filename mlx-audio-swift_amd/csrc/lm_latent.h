// lm_latent.h - mechanisms of layer-list language models (lm_blocks.hip): float32 residual stream with per-branch layer scales, latent
// attention (one cached latent + one shared rotary key part per token) under a sliding window, rotary tables with YaRN scaling.
// Every size and constant is a parameter; nothing here knows a particular model.
#pragma once
#include "common.h"
#include "lm_kernels.h"

// ---- where a producing kernel leaves the next GEMM's operand
enum { OPK_PACKED = 0,      // bf16 MFMA fragments [K/32][MT][64][8]  (decode: k_gemm_skinny)
       OPK_ROWS = 1,        // bf16 row-major [rows][ld]              (prompt pass: k_gemm_pf)
       OPK_F32 = 2 };       // float32 row-major [rows][ld]           (32-bit mode: k_gemm_f32)
struct Operand { void* p = nullptr; int kind = OPK_PACKED, ld = 0, MT = 1; };

// ---- rotary tables (host): cos / sin [positions][dims / 2], both times the magnitude factor of the scaling
struct RotarySpec {
    int dims = 0;
    double base = 10000.0;
    bool yarn = false;
    double factor = 1.0, original = 0.0, fast = 32.0, slow = 1.0;
    bool operator==(const RotarySpec& o) const {
        return dims == o.dims && base == o.base && yarn == o.yarn && factor == o.factor && original == o.original && fast == o.fast && slow == o.slow;
    }
};
void rotary_tables_host(const RotarySpec& r, int positions, std::vector<float>& cos_out, std::vector<float>& sin_out);

// ---- rows of a pass: row r belongs to sequence seq[r] (null: r) at position pos[r]; on (null: all) = 0 rows do nothing
struct RowTable { const int32_t* seq = nullptr; const int32_t* pos = nullptr; const uint8_t* on = nullptr; };

// x = rms(E[id]) * g_embed (float32 residual; g_embed null: x = E[id]), operand = rms(x) * (g_norm + g_add).  pos_cur / pos_next non-null: the decode step's position advance.
void launch_rows_embed_norm2(const bf16_t* emb, const int32_t* ids, int vocab, const bf16_t* g_embed, const bf16_t* g_norm, float* x, const Operand& h,
                             int d, int dp, float eps, int n_rows, int rows, const uint8_t* on, int32_t* pos_cur, int32_t* pos_next, hipStream_t s,
                             float g_add = 0.0f);
// x += ls1 * sum(slabs 0 .. s1 - 1) + ls2 * sum(slabs s1 .. s1 + s2 - 1); operand = rms(x) * g_norm.  Slabs [s1 + s2][slab_rows][dp] float32 (what an
// EPI_DUAL launch writes), added in slab order; s2 = 0: one branch.
struct ScaledSlabs { const float* p = nullptr; int s1 = 0, s2 = 0; const bf16_t *ls1 = nullptr, *ls2 = nullptr; };
void launch_scaled_residual_norm(const ScaledSlabs& a, int slab_rows, float* x, const bf16_t* g_norm, const Operand& h, int d, int dp, float eps, int rows,
                                 hipStream_t s);
// operand row i = rms(x[row_of[i]]) * (g_norm + g_add) (row_of null: i)
void launch_gather_norm(const float* x, const int32_t* row_of, const bf16_t* g_norm, const Operand& h, int d, int dp, float eps, int rows, hipStream_t s,
                        float g_add = 0.0f);
// block shape of the kernels that hold one row of the width per block
int row_cpt(int dp);
int row_threads(int dp, int cpt);
void row_check(int dp);

// ---- true-float32 GEMM on the packed bf16 weights (their values are exact in float32): out[m][n] = sum_k X[m][k] W[n][k], per head z
enum { F32_STORE = 0, F32_RELU2 = 1, F32_ADD_SCALED = 2, F32_SOFTCAP = 3 };
struct GemmF32 {
    const float* X; int ldx; size_t xz;            // X row stride, head stride
    const bf16_t* W; size_t wz;                    // packed [NT][KT][64][8], head stride in elements
    float* out; int ldo; size_t oz;
    int M, NT, KT, n_valid, heads = 1;
    int epi = F32_STORE;
    const bf16_t* ls = nullptr;                    // F32_ADD_SCALED: out += ls[n] * acc
    float scale = 1.0f, cap = 0.0f;                // F32_SOFTCAP: cap tanh(scale acc / cap); cap <= 0: scale acc
};
void launch_gemm_f32(const GemmF32& g, hipStream_t s);

// ---- latent attention
struct LatentDims {
    int H, n, r, v, R;          // heads, unrotated / rotated query-key dims, value dims, latent size (model sizes)
    int np, rp, vp, Rp;         // padded: np % 32, rp % 16, vp % 16, Rp % 64 (>= 128)
    int CW;                     // cache row: [latent Rp | rotary key rp | zeros], % 32
    int DK;                     // expanded query / key row: [np | rp | zeros], % 32
    int window;                 // keys a position sees, itself included; 0: all
    int rot_dims;
    float scale, eps;
};
LatentDims latent_dims(int H, int n, int r, int v, int R, int window, int rot_dims, float scale, float eps);

struct LatentRows {             // projections of a pass -> cache rows and query rows
    const float* qkv; int ld;   // [rows][H (np + rp) | Rp | rp] float32
    const bf16_t* c_norm;       // [R]
    const float *rope_cos, *rope_sin;   // [positions][rot_dims / 2]
    RowTable rows;
    void* cache;                // [sequences][Smax][CW]
    int Smax;
    void* q;                    // [rows][H][q_ld]
    int q_ld, q_rot_off;        // rotary part of a query row goes to q_rot_off; elements behind it up to q_ld are zeroed
    int with_plain;             // 1: the unrotated part is copied to the front (expanded form); 0: left to the absorb GEMM
    int f32;                    // element type of cache and q
};
void launch_latent_rows(const LatentDims& D, const LatentRows& p, int rows, hipStream_t s);
// decode, bf16: launch_latent_rows in absorbed form and q_latent = W_uk^T q in ONE launch.  uk_t: packed per head [Rp/16][np/32]
void launch_latent_absorb(const LatentDims& D, const LatentRows& p, const bf16_t* uk_t, int rows, hipStream_t s);

struct LatentAttn {
    const void* q;              // absorbed rows [rows][H][CW]
    const void* cache; int Smax;
    RowTable rows;
    void* out;                  // [rows][H][Rp] latent sums (bf16, or float32 when f32)
    int f32;
};
// any sizes, either element type
void launch_latent_attn_any(const LatentDims& D, const LatentAttn& p, int rows, hipStream_t s);
// values of the latent sums: operand[m][h v + j] = sum_R o_lat[m][h] W_uv[h][j]  (bf16; uv: packed per head, head stride uvz)
void launch_latent_values(const LatentDims& D, const bf16_t* o_lat, const bf16_t* uv, size_t uvz, const Operand& out, int rows, hipStream_t s);

// decode, bf16, matrix cores: every row's keys in S shares.  A share leaves its normalised latent sums (bf16) and (max, sum) of its scores; the
// second launch weights the shares and applies the values.
struct LatentShares { int S = 1; bf16_t* part = nullptr; float* ml = nullptr; };      // part [S][rows][H][Rp], ml [S][rows][H][2]
bool latent_decode_mfma_ok(const LatentDims& D);
int latent_decode_shares(const LatentDims& D, int rows, int Smax);
void launch_latent_attn_decode(const LatentDims& D, const LatentAttn& p, const LatentShares& sh, int rows, hipStream_t s);
void launch_latent_share_values(const LatentDims& D, const LatentShares& sh, const bf16_t* uv, size_t uvz, const Operand& out, int rows, hipStream_t s);

// prompt pass, bf16: keys and values expanded by a GEMM into kv [key rows][H np | H vp]; one block per (tile of queries of one sequence, head)
struct LatentTile { int32_t row0, n, seq, pos0, krow0, kpos0; };     // n <= LATENT_QT queries from pos0; key row of position p: krow0 + p - kpos0
#define LATENT_QT 64
struct LatentPrefill {
    const bf16_t* q;            // [rows][H][DK]
    const bf16_t* kv; int ldkv;
    const bf16_t* cache; int Smax;
    const LatentTile* tiles; int n_tiles;
    bf16_t* out; int ldo;       // [rows][ldo]
};
bool latent_prefill_mfma_ok(const LatentDims& D);
void launch_latent_attn_prefill(const LatentDims& D, const LatentPrefill& p, hipStream_t s);
