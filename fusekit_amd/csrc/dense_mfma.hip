// Matrix products of the layer-list decoder: y = x . W^T with bf16 matrices as they are stored ([n, k], rows padded to
// 64 elements), for any number of rows.
//
// Two sets of kernels.  fp32 activations (and the widths the tiles do not pay for) take plain FMA kernels.  bf16
// activations take matrix-core tiles: a block forms BM x BN outputs, its four waves WM x WN sub-tiles of 16 x 16 x 32
// instructions; 64 elements of K per step are staged in LDS, the next step's rows being on their way in registers
// while this one is multiplied.  A staged row is 128 bytes; its 16-byte pieces are XOR-swizzled by the row so that the
// sixteen rows of a fragment read hit different banks.
//
// The operand order is chosen per output layout: with the matrix rows as the first operand a lane ends up with four
// adjacent columns of one output row, with the activation rows first with four adjacent rows of one column, so row-major
// and transposed outputs both leave in whole words.
//
// Expert products take the same tile: the tile table of fusekit_route_group names the expert and the routes, rows are
// gathered through the route list, and a gate / up pair is one launch (NB = 2) whose epilogue is silu(gate) * up.
#include "column_device.hpp"

namespace fk {

namespace {

typedef __bf16 dm_bf16x8_t __attribute__((ext_vector_type(8)));
typedef float dm_f32x4_t __attribute__((ext_vector_type(4)));
typedef uint32_t dm_u32x4_t __attribute__((ext_vector_type(4)));

constexpr uint32_t kBK = 64;
constexpr int kTileThreads = 256;

enum TileOut { kOutAct = 0, kOut32 = 1, kOutT = 2 };

struct TileArgs {
    const uint16_t* x;
    const uint16_t* wa;
    const uint16_t* wb;
    void* y;
    const uint32_t* row_base;
    const uint32_t* perm;
    const uint32_t* tiles;
    const uint32_t* count;
    uint32_t ring, row_back;
    uint32_t m, n, k, ldx, ldw, ldy, x_div, tiles_m, tiles_n;
    uint64_t xb, wstride, yb;   // batch strides; wstride: per batch or per expert
    ColumnOut out;
};

__device__ __forceinline__ dm_u32x4_t lds_piece(const uint16_t* tile, uint32_t row, uint32_t piece) {
    return *reinterpret_cast<const dm_u32x4_t*>(tile + row * kBK + ((piece ^ (row & 7u)) << 3));
}

template <int BM, int BN, int WM, int WN, int NB, int OUT, bool GROUPED>
__global__ __launch_bounds__(kTileThreads) void dense_tile_kernel(const TileArgs a) {
    constexpr bool PLAIN_OUT = OUT != kOutT && NB == 1 && !GROUPED;
    constexpr int TM = BM / WM / 16, TN = BN / WN / 16;   // 16 x 16 tiles per wave
    constexpr int LA = BM / 32, LB = BN / 32;             // 16-byte pieces per thread and staged tile
    static_assert(WM * WN == 4 && BM % 32 == 0 && BN % 32 == 0, "tile shape");
    __shared__ __align__(16) uint16_t lds[2][(BM + NB * BN) * kBK];

    const uint32_t tid = threadIdx.x, lane = tid & 63u, wave = tid >> 6;
    const uint32_t wm = wave / WN, wn = wave % WN, l16 = lane & 15u, kq = lane >> 4;

    // which tile: workgroups are dealt to the eight dies in turn, so die d takes the d-th eighth of the tile list
    const uint32_t tiles_m = GROUPED ? *a.count : a.tiles_m;
    const uint32_t total = tiles_m * a.tiles_n, per = (total + 7u) / 8u;
    const uint32_t local = blockIdx.x / 8u, pid = (blockIdx.x % 8u) * per + local;
    if (local >= per || pid >= total) return;
    uint32_t mt, nt;
    if (GROUPED) {
        mt = pid / a.tiles_n;
        nt = pid - mt * a.tiles_n;
    } else {   // bands of eight row tiles walk the columns together
        const uint32_t band = pid / (8u * a.tiles_n), rem = pid - band * 8u * a.tiles_n;
        const uint32_t rows = tiles_m - band * 8u < 8u ? tiles_m - band * 8u : 8u;
        mt = band * 8u + rem % rows;
        nt = rem / rows;
    }
    const uint32_t n0 = nt * BN;
    uint32_t m0, live;
    const uint16_t *x = a.x, *wa = a.wa, *wb = a.wb;
    if (GROUPED) {
        const uint32_t* t = a.tiles + (size_t)mt * 4u;
        m0 = t[1];
        live = t[2];
        wa += (size_t)t[0] * a.wstride;
        if (NB == 2) wb += (size_t)t[0] * a.wstride;
    } else {
        m0 = mt * BM;
        live = a.m - m0 < (uint32_t)BM ? a.m - m0 : (uint32_t)BM;
        x += (size_t)blockIdx.y * a.xb;
        wa += (size_t)blockIdx.y * a.wstride;
    }
    int32_t base = 0;
    if (!GROUPED && a.ring) {
        base = (int32_t)(*a.row_base - a.row_back);
        if (base + (int32_t)(m0 + live) <= 0) return;   // every row of the tile lies before the sequence
    }

    // staging: thread t moves piece t % 8 of rows t / 8 + 32 i
    const uint32_t sr = tid >> 3, sp = tid & 7u;
    const uint16_t* pa[LA];
    const uint16_t* pb[NB][LB];
#pragma unroll
    for (int i = 0; i < LA; ++i) {
        uint32_t r = sr + 32u * i;
        r = r < live ? r : live - 1u;   // rows past the tile repeat its last one; never stored
        size_t row;
        if (GROUPED) row = a.perm[m0 + r] / a.x_div;
        else if (a.ring) row = (uint32_t)(base + (int32_t)(m0 + r)) & (a.ring - 1u);
        else row = m0 + r;
        pa[i] = x + row * a.ldx + sp * 8u;
    }
#pragma unroll
    for (int i = 0; i < LB; ++i) {
        uint32_t r = n0 + sr + 32u * i;
        r = r < a.n ? r : a.n - 1u;
        pb[0][i] = wa + (size_t)r * a.ldw + sp * 8u;
        if (NB == 2) pb[NB - 1][i] = wb + (size_t)r * a.ldw + sp * 8u;
    }
    struct Staged {
        dm_u32x4_t a[LA], b[NB][LB];
    };
    Staged r0;
    auto fetch = [&](Staged& r, uint32_t k0) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < LA; ++i) r.a[i] = *reinterpret_cast<const dm_u32x4_t*>(pa[i] + k0);
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int i = 0; i < LB; ++i) r.b[b][i] = *reinterpret_cast<const dm_u32x4_t*>(pb[b][i] + k0);
    };
    auto stage = [&](const Staged& q, uint16_t* t) __attribute__((always_inline)) {
#pragma unroll
        for (int i = 0; i < LA; ++i) {
            const uint32_t r = sr + 32u * i;
            *reinterpret_cast<dm_u32x4_t*>(t + r * kBK + ((sp ^ (r & 7u)) << 3)) = q.a[i];
        }
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int i = 0; i < LB; ++i) {
                const uint32_t r = sr + 32u * i;
                *reinterpret_cast<dm_u32x4_t*>(t + (BM + b * BN) * kBK + r * kBK + ((sp ^ (r & 7u)) << 3)) = q.b[b][i];
            }
    };

    dm_f32x4_t acc[NB][TM][TN];
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int i = 0; i < TM; ++i)
#pragma unroll
            for (int j = 0; j < TN; ++j) acc[b][i][j] = dm_f32x4_t{0.f, 0.f, 0.f, 0.f};

    const uint32_t steps = a.k / kBK;
    auto compute = [&](const uint16_t* t) __attribute__((always_inline)) {
#pragma unroll
        for (uint32_t h = 0; h < 2; ++h) {
            dm_u32x4_t fa[TM], fb[NB][TN];
#pragma unroll
            for (int i = 0; i < TM; ++i) fa[i] = lds_piece(t, wm * (BM / WM) + i * 16u + l16, h * 4u + kq);
#pragma unroll
            for (int b = 0; b < NB; ++b)
#pragma unroll
                for (int j = 0; j < TN; ++j) fb[b][j] = lds_piece(t + (BM + b * BN) * kBK, wn * (BN / WN) + j * 16u + l16, h * 4u + kq);
#pragma unroll
            for (int b = 0; b < NB; ++b)
#pragma unroll
                for (int i = 0; i < TM; ++i)
#pragma unroll
                    for (int j = 0; j < TN; ++j) {
                        const dm_bf16x8_t va = __builtin_bit_cast(dm_bf16x8_t, fa[i]), vb = __builtin_bit_cast(dm_bf16x8_t, fb[b][j]);
                        acc[b][i][j] = OUT == kOutT ? __builtin_amdgcn_mfma_f32_16x16x32_bf16(va, vb, acc[b][i][j], 0, 0, 0)
                                                    : __builtin_amdgcn_mfma_f32_16x16x32_bf16(vb, va, acc[b][i][j], 0, 0, 0);
                    }
        }
    };
    fetch(r0, 0);
    stage(r0, lds[0]);
    if constexpr (BM + NB * BN <= 128) {
        // small tiles: step s is multiplied from LDS buffer s % 2 while step s + 1 waits in registers and step s + 2 is
        // on its way; past the end the last step is requested again
        auto at = [&](uint32_t s) __attribute__((always_inline)) { return (s < steps ? s : steps - 1u) * kBK; };
        Staged r1;
        fetch(r1, at(1));
        __syncthreads();
        for (uint32_t s = 0; s < steps; s += 2u) {
            fetch(r0, at(s + 2u));
            compute(lds[0]);
            stage(r1, lds[1]);
            __syncthreads();
            if (s + 1u >= steps) break;
            fetch(r1, at(s + 3u));
            compute(lds[1]);
            stage(r0, lds[0]);
            __syncthreads();
        }
    } else {
        // large tiles hold one step in registers: two would halve the waves per SIMD
        __syncthreads();
        for (uint32_t s = 0; s < steps; ++s) {
            if (s + 1u < steps) fetch(r0, (s + 1u) * kBK);
            compute(lds[s & 1u]);
            if (s + 1u < steps) stage(r0, lds[(s + 1u) & 1u]);
            __syncthreads();
        }
    }

#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int j = 0; j < TN; ++j) {
            dm_f32x4_t v = acc[0][i][j];
            if (NB == 2) {
#pragma unroll
                for (int r = 0; r < 4; ++r) v[r] = silu(v[r]) * acc[NB - 1][i][j][r];
            }
            const uint32_t mb = wm * (BM / WM) + i * 16u, nb = n0 + wn * (BN / WN) + j * 16u;
            if (OUT == kOutT) {   // four adjacent rows of column l16
                const uint32_t n = nb + l16, mr = mb + kq * 4u;
                if (n >= a.n || mr >= live) continue;
                uint16_t* y = reinterpret_cast<uint16_t*>(a.y) + (size_t)blockIdx.y * a.yb + (size_t)n * a.ldy + m0 + mr;
                if (mr + 4u <= live && (a.ldy & 3u) == 0) {
                    *reinterpret_cast<uint2*>(y) = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
                } else {
#pragma unroll
                    for (int r = 0; r < 4; ++r)
                        if (mr + (uint32_t)r < live) y[r] = (uint16_t)f32_to_bf16_bits(v[r]);
                }
            } else {              // four adjacent columns of row l16
                const uint32_t mr = mb + l16, n = nb + kq * 4u;
                if (mr >= live || n >= a.n) continue;
                const size_t row = GROUPED ? (size_t)a.perm[m0 + mr] : (size_t)(m0 + mr);
                if (PLAIN_OUT) {
                    if (a.out.bias) {   // rows of whole fours: the planner has checked
                        const float4 b = act_load4(a.out.bias + n);
                        v[0] += b.x; v[1] += b.y; v[2] += b.z; v[3] += b.w;
                    }
                    const uint32_t fn = column_fn(a.out, n);   // one for the four columns
                    if (fn != kFnNone) {
#pragma unroll
                        for (int r = 0; r < 4; ++r) v[r] = apply_fn(fn, v[r]);
                    }
                    if (a.out.tail && n >= a.out.tail_begin) {
                        for (uint32_t r = 0; r < 4; ++r)
                            if (n + r < a.n) a.out.tail[row * a.out.ldt + n + r - a.out.tail_begin] = v[r];
                        continue;
                    }
                }
                const size_t off = (size_t)blockIdx.y * a.yb + row * a.ldy + n;
                const bool whole = n + 4u <= a.n && (a.ldy & 3u) == 0 && (a.yb & 3u) == 0;
                if (OUT == kOut32) {
                    float* y = reinterpret_cast<float*>(a.y) + off;
                    if (whole) *reinterpret_cast<float4*>(y) = make_float4(v[0], v[1], v[2], v[3]);
                    else
                        for (uint32_t r = 0; r < 4; ++r) if (n + r < a.n) y[r] = v[r];
                } else {
                    uint16_t* y = reinterpret_cast<uint16_t*>(a.y) + off;
                    if (whole) *reinterpret_cast<uint2*>(y) = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
                    else
                        for (uint32_t r = 0; r < 4; ++r) if (n + r < a.n) y[r] = (uint16_t)f32_to_bf16_bits(v[r]);
                }
            }
        }
}

// ---- plain FMA forms ----

template <typename T>
__device__ __forceinline__ size_t dense_row(const DenseArgs& a, uint32_t r) {
    return a.ring ? (size_t)((*a.row_base - a.row_back + r) & (a.ring - 1u)) : (size_t)r;
}

// A wave per column, up to eight rows of x at a time.
template <typename T>
__global__ __launch_bounds__(256) void dense_few_kernel(const DenseArgs a) {
    const uint32_t lane = threadIdx.x & 63u, n = blockIdx.x * 4u + (threadIdx.x >> 6), r0 = blockIdx.y * 8u;
    if (n >= a.n) return;
    const T* x = reinterpret_cast<const T*>(a.x) + (size_t)blockIdx.z * a.xb;
    const uint16_t* w = a.w + (size_t)blockIdx.z * a.wb + (size_t)n * a.ldw;
    const uint32_t rows = a.m - r0 < 8u ? a.m - r0 : 8u;
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    for (uint32_t c = lane * 4u; c < a.k; c += 256u) {
        const float4 wv = act_load4(w + c);
#pragma unroll
        for (uint32_t r = 0; r < 8; ++r) {
            if (r >= rows) break;
            const float4 v = act_load4(x + dense_row<T>(a, r0 + r) * a.ldx + c);
            acc[r] = fmaf(v.x, wv.x, acc[r]); acc[r] = fmaf(v.y, wv.y, acc[r]);
            acc[r] = fmaf(v.z, wv.z, acc[r]); acc[r] = fmaf(v.w, wv.w, acc[r]);
        }
    }
#pragma unroll
    for (uint32_t r = 0; r < 8; ++r) {
        const float v = column_value(a.out, n, wave_sum(acc[r]));
        if (lane == 0 && r < rows) {
            const size_t off = (size_t)blockIdx.z * a.yb + (size_t)(r0 + r) * a.ldy + n;
            if (a.out.tail && n >= a.out.tail_begin) a.out.tail[(size_t)(r0 + r) * a.out.ldt + n - a.out.tail_begin] = v;
            else if (a.y32) reinterpret_cast<float*>(a.y)[off] = v;
            else act_store(reinterpret_cast<T*>(a.y) + off, v);
        }
    }
}

// 64 x 64 outputs per block, 16 of K per step, 4 x 4 per thread.
__global__ __launch_bounds__(256) void dense_f32_kernel(const DenseArgs a) {
    __shared__ float xs[16][68], ws[16][68];
    const uint32_t tid = threadIdx.x, tx = tid & 15u, ty = tid >> 4;
    const uint32_t m0 = blockIdx.y * 64u, n0 = blockIdx.x * 64u;
    const float* x = reinterpret_cast<const float*>(a.x) + (size_t)blockIdx.z * a.xb;
    const uint16_t* w = a.w + (size_t)blockIdx.z * a.wb;
    const uint32_t lr = tid >> 2, lc = (tid & 3u) * 4u;
    const uint32_t mr = m0 + lr < a.m ? m0 + lr : a.m - 1u, nr = n0 + lr < a.n ? n0 + lr : a.n - 1u;
    const float* px = x + dense_row<float>(a, mr) * a.ldx + lc;
    const uint16_t* pw = w + (size_t)nr * a.ldw + lc;
    float acc[4][4] = {};
    for (uint32_t k0 = 0; k0 < a.k; k0 += 16u) {
        const float4 xv = act_load4(px + k0), wv = act_load4(pw + k0);
        __syncthreads();
        xs[lc][lr] = xv.x; xs[lc + 1][lr] = xv.y; xs[lc + 2][lr] = xv.z; xs[lc + 3][lr] = xv.w;
        ws[lc][lr] = wv.x; ws[lc + 1][lr] = wv.y; ws[lc + 2][lr] = wv.z; ws[lc + 3][lr] = wv.w;
        __syncthreads();
#pragma unroll
        for (int k = 0; k < 16; ++k) {
            float xr[4], wr[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) { xr[i] = xs[k][ty * 4u + i]; wr[i] = ws[k][tx * 4u + i]; }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xr[i], wr[j], acc[i][j]);
        }
    }
    float* y = reinterpret_cast<float*>(a.y) + (size_t)blockIdx.z * a.yb;
    for (uint32_t i = 0; i < 4; ++i)
        for (uint32_t j = 0; j < 4; ++j) {
            const uint32_t m = m0 + ty * 4u + i, n = n0 + tx * 4u + j;
            if (m >= a.m || n >= a.n) continue;
            const float v = column_value(a.out, n, acc[i][j]);
            if (a.out.tail && n >= a.out.tail_begin) a.out.tail[(size_t)m * a.out.ldt + n - a.out.tail_begin] = v;
            else y[(size_t)m * a.ldy + n] = v;
        }
}

template <int BM, int BN, int WM, int WN, int NB, bool GROUPED>
const void* tile_func(int out) {
    if (out == kOut32) return (const void*)&dense_tile_kernel<BM, BN, WM, WN, NB, kOut32, GROUPED>;
    if (out == kOutT) return (const void*)&dense_tile_kernel<BM, BN, WM, WN, NB, kOutT, GROUPED>;
    return (const void*)&dense_tile_kernel<BM, BN, WM, WN, NB, kOutAct, GROUPED>;
}

}  // namespace

fk_status plan_dense(const DenseArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "dense: act must be 16 or 32");
    if (!a.x || !a.w || !a.y || !a.m || !a.n || !a.k || !a.batch) return set_error(FK_ERR_INVALID, "dense: bad arguments");
    if (a.k % kRowPad || a.ldx % 4 || a.ldw % 8 || (a.batch == 1 && a.ldx < a.k && a.m > 1) || a.ldw < a.k)
        return set_error(FK_ERR_INVALID, "dense: k must be a multiple of 64 within padded rows");
    if (a.ring && ((a.ring & (a.ring - 1)) || !a.row_base || a.m > a.ring)) return set_error(FK_ERR_INVALID, "dense: the ring must be a power of two of at least m rows");
    if (a.batch > 65535) return set_error(FK_ERR_UNSUPPORTED, "dense: at most 65535 batches");
    if (a.transposed && (act != 16 || a.y32)) return set_error(FK_ERR_UNSUPPORTED, "dense: transposed outputs are bf16");
    const ColumnOut& o = a.out;
    if (o.bias || o.tail || o.fn || o.fn2) {
        if (a.transposed || a.batch != 1) return set_error(FK_ERR_UNSUPPORTED, "dense: column functions go with one row-major product");
        if (o.fn > kFnMax || o.fn2 > kFnMax || o.begin % 4 || o.end % 4 || o.begin2 % 4 || (o.tail && (o.tail_begin % 4 || o.tail_begin > a.n || o.ldt < a.n - o.tail_begin)))
            return set_error(FK_ERR_INVALID, "dense: column functions start at multiples of four columns");
        if (o.bias && act == 16 && (a.n % 4 || ((uintptr_t)o.bias & 7u))) return set_error(FK_ERR_INVALID, "dense: biases come in fours");
    }
    out->shmem = 0;
    out->block = dim3(256, 1, 1);
    if (act == 32 || (a.m <= 8 && !a.transposed)) {
        if (a.m <= 8) {
            out->func = act == 16 ? (const void*)&dense_few_kernel<uint16_t> : (const void*)&dense_few_kernel<float>;
            out->grid = dim3((a.n + 3u) / 4u, (a.m + 7u) / 8u, a.batch);
        } else {
            if ((a.m + 63u) / 64u > 65535) return set_error(FK_ERR_UNSUPPORTED, "dense: too many rows");
            out->func = (const void*)&dense_f32_kernel;
            out->grid = dim3((a.n + 63u) / 64u, (a.m + 63u) / 64u, a.batch);
        }
        out->set_args(a);
        return FK_OK;
    }
    if (a.ldx % 8 || a.xb % 8 || a.wb % 8) return set_error(FK_ERR_INVALID, "dense: rows must be 16-byte aligned");
    TileArgs t;
    memset(&t, 0, sizeof(t));
    t.x = (const uint16_t*)a.x; t.wa = a.w; t.y = a.y; t.row_base = a.row_base; t.ring = a.ring; t.row_back = a.row_back;
    t.m = a.m; t.n = a.n; t.k = a.k; t.ldx = a.ldx; t.ldw = a.ldw; t.ldy = a.ldy;
    t.xb = a.xb; t.wstride = a.wb; t.yb = a.yb;
    t.out = a.out;
    const int kind = a.transposed ? kOutT : (a.y32 ? kOut32 : kOutAct);
    auto blocks = [&](uint32_t bm, uint32_t bn) { return (uint64_t)((a.m + bm - 1) / bm) * ((a.n + bn - 1) / bn) * a.batch; };
    uint32_t bm, bn;
    if (a.m <= 32 || blocks(64, 64) < 128) { bm = 32; bn = 64; out->func = tile_func<32, 64, 1, 4, 1, false>(kind); }
    else if (blocks(128, 128) >= 192) { bm = 128; bn = 128; out->func = tile_func<128, 128, 2, 2, 1, false>(kind); }
    else { bm = 64; bn = 64; out->func = tile_func<64, 64, 2, 2, 1, false>(kind); }
    t.tiles_m = (a.m + bm - 1) / bm;
    t.tiles_n = (a.n + bn - 1) / bn;
    const uint64_t g = ((uint64_t)t.tiles_m * t.tiles_n + 7) / 8 * 8;
    if (g > 0x7fffffffull) return set_error(FK_ERR_UNSUPPORTED, "dense: too many tiles");
    out->grid = dim3((uint32_t)g, a.batch, 1);
    out->set_args(t);
    return FK_OK;
}

fk_status plan_experts_grouped(const ExpertArgs& a, Launch* out) {
    if (!a.tiles || !a.count) return set_error(FK_ERR_INVALID, "experts: the grouped form needs the tile table");
    if (a.ldx % 8 || a.ldw % 8 || a.ldy % 4) return set_error(FK_ERR_INVALID, "experts: rows must be padded");
    TileArgs t;
    memset(&t, 0, sizeof(t));
    t.x = (const uint16_t*)a.x; t.wa = a.wa; t.wb = a.wb; t.y = a.y; t.perm = a.perm; t.tiles = a.tiles; t.count = a.count;
    t.n = a.n; t.k = a.k; t.ldx = a.ldx; t.ldw = a.ldw; t.ldy = a.ldy; t.x_div = a.x_div;
    t.wstride = (uint64_t)a.n * a.ldw;
    uint32_t bn;
    if (a.wb) {
        if (a.tile_rows == 32) { bn = 64; out->func = (const void*)&dense_tile_kernel<32, 64, 1, 4, 2, kOutAct, true>; }
        else if (a.tile_rows == 64) { bn = 64; out->func = (const void*)&dense_tile_kernel<64, 64, 2, 2, 2, kOutAct, true>; }
        else if (a.tile_rows == 128) { bn = 64; out->func = (const void*)&dense_tile_kernel<128, 64, 2, 2, 2, kOutAct, true>; }
        else return set_error(FK_ERR_UNSUPPORTED, "experts: tiles of 32, 64 or 128 routes");
    } else {
        if (a.tile_rows == 32) { bn = 64; out->func = (const void*)&dense_tile_kernel<32, 64, 1, 4, 1, kOutAct, true>; }
        else if (a.tile_rows == 64) { bn = 64; out->func = (const void*)&dense_tile_kernel<64, 64, 2, 2, 1, kOutAct, true>; }
        else if (a.tile_rows == 128) { bn = 128; out->func = (const void*)&dense_tile_kernel<128, 128, 2, 2, 1, kOutAct, true>; }
        else return set_error(FK_ERR_UNSUPPORTED, "experts: tiles of 32, 64 or 128 routes");
    }
    t.tiles_m = a.max_tiles;
    t.tiles_n = (a.n + bn - 1) / bn;
    const uint64_t g = ((uint64_t)a.max_tiles * t.tiles_n + 7) / 8 * 8;
    if (g > 0x7fffffffull) return set_error(FK_ERR_UNSUPPORTED, "experts: too many tiles");
    out->grid = dim3((uint32_t)g, 1, 1);
    out->block = dim3(kTileThreads, 1, 1);
    out->shmem = 0;
    out->set_args(t);
    return FK_OK;
}

}  // namespace fk
