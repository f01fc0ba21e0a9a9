// Planners and argument blocks of the layer-list decoder: a decoder whose layers are described one by one (a mixer
// and an optional feed-forward each), with a 32-bit residual stream.
//
// Conventions shared by all of them.
//  * `act` is the width of an activation element: 16 (bf16) or 32 (fp32).  The same kernels serve both; matrices are
//    bf16 in either case (they are stored so) and accumulation is fp32.
//  * Rows of matrices and of activations are padded with zeros to a multiple of kRowPad elements (`ld*` is the padded
//    length), so that no kernel needs a tail along K.  Buffers start as zeros and kernels write valid columns only.
//  * Positions are device words: row r of a pass is position *offset + r.
#pragma once
#include "fk_host.hpp"

namespace fk {

constexpr uint32_t kRowPad = 64;

// x += mixer output + feed-forward output (+ a constant vector), then up to two norms of the new x: RMS norms, or layer
// norms where a bias is given.
struct ResidualNormArgs {
    float* x;               // [rows, ldx]
    const float* mix;       // [parts][rows, ldx] (a product in parts of its sum) or null
    const void* routes;     // [rows * top, ldx] expert outputs (act) or null
    const float* weight;    // [rows, top] route weights
    const uint32_t* index;  // [rows, top] chosen experts; >= experts: the identity, whose output is prev
    const void* prev;       // [rows, ldx] the feed-forward's input (act)
    const uint16_t* step;   // [width] added as well, or null
    const uint16_t* w1;     // norm weights [ldx] or null
    const uint16_t* w2;
    const uint16_t* b1;     // layer norm's bias [ldx], or null: RMS norm (the second norm is always one)
    void* h1;               // [rows, ldx] (act)
    void* h2;
    void* copy;             // [rows, ldcopy] (act): the new x itself, or null
    uint32_t rows, width, ldx, top, experts, ldcopy, parts;
    float eps;
};
fk_status plan_residual_norm(const ResidualNormArgs& a, uint32_t act, Launch* out);

// y[r] = x[r] / rms(x[r]) * w in `groups` equal parts, optionally of the gated row x * silu(z).
struct GroupNormArgs {
    const void* x;      // [rows, ldx]; fp32 when x32, else act
    const void* z;      // [rows, ldz] (act) or null
    const uint16_t* w;  // [width]
    void* y;            // [rows, ldy] (act)
    uint32_t rows, width, groups, ldx, ldz, ldy, x32;
    float eps;
};
fk_status plan_group_norm(const GroupNormArgs& a, uint32_t act, Launch* out);

// What becomes of a product's columns before they are stored.  All bounds are multiples of four columns.
enum ColumnFn : uint32_t {
    kFnNone = 0,
    kFnRelu2 = 1,   // the square of relu
    kFnGelu = 2,    // gelu, tanh form
    kFnMax = 2,
};
struct ColumnOut {
    const uint16_t* bias;       // [n] added first, or null
    float* tail;                // columns tail_begin .. are stored here as fp32 instead, or null
    uint32_t fn, begin, end;    // function of columns begin .. end - 1
    uint32_t fn2, begin2;       // function of columns begin2 ..
    uint32_t tail_begin, ldt;
};

// Token rows: x = scale * table[token] (+ a row of a second table, chosen by a hash of the token and the one before it).
struct EmbedRowsArgs {
    const uint32_t* tokens;   // [rows]
    const uint16_t* table;    // [vocab, ldw]
    const uint16_t* pairs;    // [buckets + 1, ldw] or null; the last row is for the first token of a sequence
    uint32_t* prev;           // the token before the pass; becomes the last one of it
    const uint32_t* offset;
    float* x;                 // [rows, ldx]
    void* copy;               // [rows, ldcopy] (act) or null
    uint32_t rows, width, vocab, buckets, mul_prev, mul_cur, ldw, ldx, ldcopy;
    float scale;
};
fk_status plan_embed_rows(const EmbedRowsArgs& a, uint32_t act, Launch* out);

// y[r, h] = x[r, h] / rms(x[r, h]) * w * sigmoid(z[r, h]) per head of `dim` elements (`ld` padded).
struct HeadNormArgs {
    const float* x;      // [rows, ldx]
    const void* z;       // [rows, ldz] (act)
    const uint16_t* w;   // [ld], shared by the heads
    void* y;             // [rows, ldy] (act)
    uint32_t rows, heads, dim, ld, ldx, ldz, ldy;
    float eps;
};
fk_status plan_head_norm(const HeadNormArgs& a, uint32_t act, Launch* out);

// y[b][m, n] = x[b][m, k] . w[b][n, k]^T.
struct DenseArgs {
    const void* x;
    const uint16_t* w;
    void* y;                   // fp32 when y32, else act
    const uint32_t* row_base;  // with ring: row r of x is row (*row_base + r - row_back) & (ring - 1)
    uint32_t ring, row_back;   // ring 0: plain rows; rows of negative position are skipped tile by tile
    uint32_t m, n, k;          // k: padded length of the dot products
    uint32_t ldx, ldw, ldy, batch;
    uint64_t xb, wb, yb;       // elements between batches
    uint32_t y32, transposed;  // transposed: y[b][n, m] (bf16 matrix-core form only)
    ColumnOut out;             // row-major outputs of plain rows only
};
fk_status plan_dense(const DenseArgs& a, uint32_t act, Launch* out);

// Router: softmax over all outputs, choice by score + correction, weights = chosen scores over their sum.
struct RouteArgs {
    const float* logits;         // [rows, ldl]
    const uint16_t* correction;  // [outputs]
    uint32_t* index;             // [rows, top]
    float* weight;               // [rows, top]
    uint32_t rows, outputs, top, ldl;
};
fk_status plan_route_rows(const RouteArgs& a, Launch* out);
constexpr uint32_t kMaxRouterOutputs = 1024, kMaxRouterTop = 64;

// The routes of a pass grouped by expert for the tiled expert products: `perm` lists routes expert by expert,
// `tiles` holds (expert, first place in perm, routes) per tile of `tile_rows` routes, `count` the number of tiles.
struct RouteGroupArgs {
    const uint32_t* index;  // [routes]
    uint32_t* perm;         // [routes]
    uint32_t* tiles;        // [max_tiles][4]
    uint32_t* count;
    uint32_t routes, experts, tile_rows, max_tiles;
};
fk_status plan_route_group(const RouteGroupArgs& a, Launch* out);

// One matrix (or a gate / up pair with silu(gate) * up) of the chosen experts.  Route r reads row r / x_div of x.
struct ExpertArgs {
    const void* x;          // [.., ldx] (act)
    const uint16_t* wa;     // [experts][n, ldw]
    const uint16_t* wb;     // the up matrices, or null
    const uint32_t* index;  // [routes]
    void* y;                // [routes, ldy] (act)
    const uint32_t* perm;   // grouped form (bf16): from fusekit_route_group
    const uint32_t* tiles;
    const uint32_t* count;
    uint32_t routes, experts, n, k, ldx, ldw, ldy, x_div, tile_rows, max_tiles;
};
fk_status plan_experts(const ExpertArgs& a, uint32_t act, Launch* out);

// ---- latent attention ----
// The cache of one layer run is a ring of rows [latent, padded | rotated key part, padded] (act); position p lives in
// row p & (ring - 1).  A pass writes its rows, then reads the window behind each of its own positions, so a ring of
// window + rows - 1 positions is enough whatever the length of the sequence.
struct LatentStoreArgs {
    const float* kv;          // [rows, ldkv]: latent | key part
    const uint16_t* norm;     // [rank]
    const double* freq;       // [rot / 2] radians per position
    void* cache;              // [ring, ldc]
    void* q;                  // rows of ldq (act), head h at h * hs: the rot part, at dim_ld, is rotated in place
    const uint32_t* offset;
    uint32_t rows, rank, ldkv, ldc, rank_ld, ring, heads, hs, dim_ld, rot, rot_dims, ldq;
    float eps;
};
fk_status plan_latent_store(const LatentStoreArgs& a, uint32_t act, Launch* out);

// Attention in the latent space, one query row after the other: qa = W_uk^T q per head meets the cached latents, the
// weighted sum of latents is left to W_uv.
struct LatentAttnArgs {
    const void* qa;         // [rows, heads, rank_ld]; fp32 when act is 32, else bf16
    const void* q;          // [rows, ldq] (act), rotated
    const void* cache;      // [ring, ldc]
    const uint16_t* sink;   // [heads]
    void* out;              // [rows, heads, rank_ld] (act)
    float* part;            // split form: [rows, splits, heads, rank_ld + 2]
    const uint32_t* offset;
    uint32_t rows, heads, hs, dim_ld, rot, rank, rank_ld, ldc, ldq, ring, window, splits;
    float scale;
};
fk_status plan_latent_attn(const LatentAttnArgs& a, uint32_t act, Launch* out);

// The same for a few rows on the matrix cores (bf16): the window in `splits` spans of whole 64-position tiles, partial
// rows [rows, splits, heads, rank_ld + 2] = latent sums | maximum | sum of weights.
struct LatentSplitArgs {
    const uint16_t* qa;
    const uint16_t* q;
    const uint16_t* cache;
    const uint16_t* sink;
    uint16_t* out;          // [rows, heads, rank_ld] when combined here
    float* part;
    const float* tab;       // [rot_dims] cos, sin per pair: rotates q while it is read; null: q is rotated already
    const uint32_t* offset;
    uint32_t rows, heads, hs, dim_ld, rot, rot_dims, rank_ld, ldc, ldq, ring, window, splits, span;
    float scale;
};
constexpr uint32_t kMaxSplits = 64;
bool latent_split_supported(uint32_t rank_ld, uint32_t ldc);
fk_status plan_latent_split(LatentSplitArgs& a, bool combine, Launch* out);

// Attention of a pass with keys and values formed from the latents (bf16): row 0 of k / column 0 of vt is position
// *offset - (window - 1).
struct LatentPrefillArgs {
    const uint16_t* q;      // [rows, ldq], rotated; a head is [dim_ld | rot_ld], zero padded
    const uint16_t* k;      // [window - 1 + rows, ldk]: unrotated key parts, dim_ld per head
    const uint16_t* vt;     // [heads * vdim_ld, ldv]: values, transposed
    const uint16_t* cache;  // [ring, ldc]: the rotated key parts
    const uint16_t* sink;
    uint16_t* out;          // [rows, ldo]: heads * vdim_ld
    const uint32_t* offset;
    uint32_t rows, heads, dim_ld, rot_ld, vdim_ld, ldq, ldk, ldv, ldo, ldc, rank_ld, ring, window;
    float scale;
};
bool latent_prefill_supported(uint32_t dim_ld, uint32_t rot_ld, uint32_t vdim_ld);
fk_status plan_latent_prefill(const LatentPrefillArgs& a, Launch* out);

// ---- state-space mixer ----
// conv: y[r, c] = f(b[c] + sum_k w[c, k] u[r - taps + 1 + k, c]), f = silu or nothing; rows before the pass come from
// `hist` [taps, ldh], where position p lies in row p % taps.
struct SsmConvArgs {
    const void* u;      // [rows, ldu] (act), at the first convolved column
    const uint16_t* w;  // [channels, taps]
    const uint16_t* b;  // [channels] or null
    void* hist;         // (act)
    void* y;            // [rows, ldy] (act)
    const uint32_t* offset;
    uint32_t rows, channels, taps, ldu, ldy, ldh;
    uint32_t linear, update;   // linear: no silu; update: the history takes the rows of this pass (else the scan does it)
};
fk_status plan_ssm_conv(const SsmConvArgs& a, uint32_t act, Launch* out);

// The recurrence over the rows of a pass, row after row, and the update of the convolution's history.
struct SsmScanArgs {
    const void* xbc;          // [rows, ldx] (act) after the convolution: x | B | C
    const float* dt;          // [rows, lddt] before bias and softplus
    const uint16_t* dt_bias;  // [heads]
    const uint16_t* a_log;
    const uint16_t* d;
    float* state;             // [heads][vdim][state_ld]
    void* y;                  // [rows, ldy] (act)
    const void* u;            // [rows, ldu] (act) and hist [taps, ldh]: the rows to remember
    void* hist;
    const uint32_t* offset;
    uint32_t rows, heads, groups, n, p, state_ld, ldx, lddt, ldy, ldu, ldh, channels, taps;
};
fk_status plan_ssm_scan(const SsmScanArgs& a, uint32_t act, Launch* out);
constexpr uint32_t kMaxSsmState = 256;

// The same in chunks of 64 tokens on the matrix cores (bf16).
struct SsmChunkArgs {
    const uint16_t* xbc;
    const float* dt;
    const uint16_t* dt_bias;
    const uint16_t* a_log;
    const uint16_t* d;
    float* state;
    uint16_t* y;
    const uint16_t* u;
    uint16_t* hist;
    const uint32_t* offset;
    float* chunks;  // [chunks][heads][p][state_ld]
    float* decay;   // [chunks][heads]
    uint32_t rows, heads, groups, n, p, state_ld, ldx, lddt, ldy, ldu, ldh, channels, taps;
};
constexpr uint32_t kSsmChunk = 64;
bool ssm_chunk_supported(uint32_t heads, uint32_t p, uint32_t n);
fk_status plan_ssm_chunk(const SsmChunkArgs& a, Launch* out);

// ---- grouped-query attention ----
// One launch between the joint input projection and the attention of a pass: RMS norm of the whole query row and of the
// whole key row (all heads at once), rotation, the new cache rows.  The values are the keys as they were projected.
// Heads are padded to dim_ld elements; caches are [kv_heads][capacity][dim_ld].
struct QkStoreArgs {
    const void* u;            // [rows, ldu] (act): keys at column k0, queries at column q0
    const uint16_t* wq;       // [heads * dim_ld] norm weights
    const uint16_t* wk;       // [kv_heads * dim_ld]
    const double* freq;       // [rot_dims / 2] radians per position
    void* q;                  // [rows, heads * dim_ld] (act)
    void* cache_k;
    void* cache_v;
    const uint32_t* offset;
    uint32_t rows, heads, kv_heads, dim, dim_ld, rot_dims, ldu, k0, q0, capacity;
    float eps, mag;           // mag: factor of cos and sin
};
fk_status plan_qk_store(const QkStoreArgs& a, uint32_t act, Launch* out);

// Causal attention of the rows of a pass, any head width, one workgroup per (head, row).
struct GqaRowsArgs {
    const void* q;            // [rows, heads * dim_ld] (act)
    const void* cache_k;
    const void* cache_v;
    const uint32_t* offset;
    void* out;                // [rows, ldo] (act)
    uint32_t rows, heads, kv_heads, dim_ld, capacity, ldo;
    float scale;
};
constexpr uint32_t kMaxGqaDim = 512;
fk_status plan_gqa_rows(const GqaRowsArgs& a, uint32_t act, Launch* out);

// ---- gated delta rule with one decay per key channel ----
// Head h of `heads` has its own state, values and decays and shares queries and keys of head h / (heads / kv_heads).
// Head widths are padded to whole 32s (dim_ld, vdim_ld); the padding holds zeros.
//
// prep: unit vectors of the convolved queries (times dim^-1/2) and keys, log2 of the decays, step sizes.
struct DeltaPrepArgs {
    const void* xc;           // [rows, ldx] (act) after the convolution: q | k | v
    const uint16_t* dt_bias;  // [heads * dim_ld]
    const uint16_t* a_log;    // [heads]
    float* decay;             // [rows, heads * dim_ld]: the projection before bias and softplus; becomes log2 of the decay
    float* beta;              // [rows, ldb]: before the sigmoid; becomes the step size
    float* qk;                // [rows, 2 * kv_heads * dim_ld]
    uint32_t rows, heads, kv_heads, dim, dim_ld, ldx, ldb;
};
fk_status plan_delta_prep(const DeltaPrepArgs& a, uint32_t act, Launch* out);

// The recurrence over the rows of a pass, row after row.
struct DeltaScanArgs {
    const float* qk;
    const float* decay;
    const float* beta;
    const void* v;            // [rows, ldx] (act), at the first value column
    float* state;             // [heads][vdim_ld][state_ld]
    float* o;                 // [rows, heads * vdim_ld]
    uint32_t rows, heads, kv_heads, dim_ld, vdim_ld, state_ld, ldx, ldb;
};
fk_status plan_delta_scan(const DeltaScanArgs& a, uint32_t act, Launch* out);

// The same in chunks of 64 tokens on the matrix cores (bf16); `work`: delta_chunk_work_bytes; o has whole chunks of rows.
struct DeltaChunkArgs {
    const float* qk;
    const float* decay;
    const float* beta;
    const uint16_t* v;
    float* state;
    float* o;
    void* work;
    uint32_t rows, heads, kv_heads, dim_ld, vdim_ld, state_ld, ldx, ldb;
};
constexpr uint32_t kDeltaChunk = 64;
bool delta_chunk_supported(uint32_t dim_ld, uint32_t vdim_ld);
uint64_t delta_chunk_work_bytes(uint32_t rows, uint32_t heads, uint32_t dim_ld, uint32_t vdim_ld);
fk_status plan_delta_chunk(const DeltaChunkArgs& a, Launch* out);

// ---- real-gated linear recurrent unit ----
// S <- a S + sqrt(1 - a^2) i u, log a = -8 r softplus(lam), r and i sigmoids of block-diagonal products; the output is
// S times the gate branch, in its place.  `width` counts padded channels.
struct LruScanArgs {
    const void* u;            // [rows, ldx] (act) after the convolution
    const float* gates;       // [rows, 2 * width]: per block of `block` channels its r, then its i, before bias and sigmoid
    const uint16_t* rb;       // [width]
    const uint16_t* ib;
    const uint16_t* lam;
    float* state;             // [width]
    void* y;                  // [rows, ldy] (act): the gate branch in, the output out
    float* carry;             // [chunks][2][width]: product of decays and end of every chunk but the last, a copy of the state
    uint32_t rows, width, block, ldx, ldy;
};
constexpr uint32_t kLruChunk = 32;
fk_status plan_lru_scan(const LruScanArgs& a, uint32_t act, Launch* out);

}  // namespace fk
