// Argument blocks of the fused decode launches of the layer-list decoder (layer_decode.hip).  A job whose first pointer
// is null is absent; the planners fill in the workgroup ranges.
#pragma once
#include <algorithm>

#include "layered.hpp"

namespace fk {

constexpr uint32_t kMaxGemvJobs = 2, kMaxGateGroups = 64;

// How the input row of a product is formed.
enum RowMode : uint32_t {
    kRowPlain = 0,    // bf16, as it is
    kRowNorm = 1,     // fp32 (+ a bf16 vector), RMS norm or (with a bias) layer norm
    kRowGated = 2,    // bf16 x * silu(z), RMS norm in groups
    kRowCombine = 3,  // partial rows of the split attention, per head
    kRowJoin = 4,     // an fp32 row and behind it a bf16 one, half of k each
};

struct GemvJob {
    const void* x;
    const void* x2;       // kRowNorm: vector added first, or null; kRowGated: z; kRowJoin: the second row
    const uint16_t* nw;   // norm weights; kRowCombine: the sinks
    const uint16_t* nb;   // kRowNorm: layer norm's bias, or null
    const uint16_t* w;
    void* y;              // bf16 outputs of rows below n_act
    float* y32;           // fp32 outputs of rows n_act ..
    uint16_t* keep;       // kRowNorm: the normalised row is also written here
    uint32_t mode, n, k, ldw, width, n_act;
    uint32_t rows_per_head, x_head, y_head;   // per-head products: head h (of n / rows_per_head) reads x + h * x_head, writes y + h * y_head
    uint32_t groups, splits, heads, pl, vec;
    float eps;
    ColumnOut out;        // biases and functions of the outputs (its tail is y32)
    uint32_t first, blocks, rows_per_block, blocks_per_head;
};
struct PairJob {
    const uint16_t* x;
    const uint16_t* wa;   // [experts][n, ldw]
    const uint16_t* wb;
    const uint32_t* index;
    uint16_t* y;          // [top, ldy]
    uint32_t n, k, ldw, ldy, top, experts;
    uint32_t first, blocks, rows_per_block, blocks_per_slot;
};
struct RouteJob {
    const float* logits;
    const uint16_t* correction;
    uint32_t* index;
    float* weight;
    uint32_t outputs, top, first, blocks;
};
struct StoreJob {
    const float* kv;
    const uint16_t* norm;
    const double* freq;
    uint16_t* cache;
    float* tab;           // [rot_dims] the rotation of this position (cos, sin per pair), for the queries
    const uint32_t* offset;
    uint32_t rank, rank_ld, ldc, ring, rot, rot_dims;
    float eps;
    uint32_t first, blocks;
};
struct ScanJob {
    const uint16_t* u;    // raw rows: x | B | C
    const float* dt;
    const uint16_t* w;    // convolution
    const uint16_t* b;
    const uint16_t* dt_bias;
    const uint16_t* a_log;
    const uint16_t* d;
    float* state;
    uint16_t* hist;
    uint16_t* y;
    const uint32_t* offset;
    uint32_t heads, groups, n, p, state_ld, ldh, taps, first, blocks;
};
// One token of a gated delta rule: convolution, unit vectors, decays (their second projection included), state.
struct DeltaJob {
    const uint16_t* u;    // raw rows: q | k | v
    const uint16_t* a1;   // [rank_ld] first projection of the decays
    const float* beta;    // [heads] before the sigmoid
    const uint16_t* w;    // convolution
    const uint16_t* a2;   // [heads * dim_ld, rank_ld]
    const uint16_t* dt_bias;
    const uint16_t* a_log;
    const uint32_t* offset;
    float* state;
    uint16_t* hist;
    float* o;             // [heads * vdim_ld]
    uint32_t heads, kv_heads, dim, dim_ld, vdim_ld, state_ld, rank_ld, ldh, taps, first, blocks;
};
// One token of a gated linear recurrence: convolution, gates, state, output.
struct LruJob {
    const uint16_t* u;    // [width] raw
    const uint16_t* w;    // convolution
    const uint16_t* b;
    const uint16_t* gates;   // [blocks][r | i][block, block]
    const uint16_t* rb;
    const uint16_t* ib;
    const uint16_t* lam;
    const uint32_t* offset;
    float* state;
    uint16_t* hist;
    uint16_t* y;          // [width] the gate branch, replaced by the output
    uint32_t width, block, ldh, taps, first, blocks, blocks_per_part;
};
constexpr uint32_t kLruRows = 16;   // channels per workgroup
struct LayerJobsArgs {
    GemvJob gemv[kMaxGemvJobs];
    PairJob pair;
    RouteJob route;
    StoreJob store;
    ScanJob scan;
    DeltaJob delta;
    LruJob lru;
};
fk_status plan_layer_jobs(LayerJobsArgs& a, Launch* out);

struct LayerOutArgs {
    float* x;               // [n], updated
    const float* mix;       // the mixer's output, or null
    const uint16_t* att;    // the output projection's input and matrix, or null
    const uint16_t* wo;     // [n, ldo]
    const uint16_t* eh;     // [top, kf]
    const uint16_t* wd;     // [experts][n, kf]
    const uint32_t* index;
    const float* weight;
    const uint16_t* h2;     // the feed-forward's input
    const uint16_t* step;   // added as well, or null
    // with ho: the first heads * hld elements of the output projection's input are formed here, ho / rms * hw * sigmoid(hz)
    // per head, the rest comes from att
    const float* ho;
    const uint16_t* hz;
    const uint16_t* hw;
    uint32_t n, ko, ldo, kf, top, experts, max_items, heads, hdim, hld;
    float heps;
};
fk_status plan_layer_out(LayerOutArgs& a, Launch* out);

}  // namespace fk
