// Real-gated linear recurrent unit: per channel
//     S <- a S + sqrt(1 - a^2) i u,   log a = -8 r softplus(lam),   r, i = sigmoid(block-diagonal products)
// and the output S times the gate branch.  A channel is independent of all others and its recurrence is linear, so a pass
// runs in chunks of 32 tokens side by side: every chunk's product of decays and its end from a zero state, then every
// chunk once more from the state its predecessors leave, which each thread forms from their ends.
#include "lru_device.hpp"

namespace fk {

namespace {

// One channel's constants, and its inputs for half a chunk.
template <typename T>
struct LruColumn {
    static constexpr uint32_t kHalf = kLruChunk / 2;
    struct Rows {
        float u[kHalf], r[kHalf], i[kHalf], y[kHalf];
    };
    const LruScanArgs& a;
    const T* u;
    const float* gr;
    float rb, ib, rate;

    __device__ LruColumn(const LruScanArgs& args, uint32_t c)
        : a(args), u(reinterpret_cast<const T*>(args.u) + c), gr(args.gates + (size_t)(c / args.block) * 2u * args.block + c % args.block),
          rb(bf16_bits_to_f32(args.rb[c])), ib(bf16_bits_to_f32(args.ib[c])), rate(lru_rate(args.lam[c])) {}

    // Requests only, all of them in flight together; rows past the pass repeat its last one.
    template <bool GATE>
    __device__ __forceinline__ void fetch(Rows& x, uint32_t r0, const T* y) const {
#pragma unroll
        for (uint32_t e = 0; e < kHalf; ++e) {
            const uint32_t r = r0 + e < a.rows ? r0 + e : a.rows - 1u;
            x.u[e] = act_load(u + (size_t)r * a.ldx);
            x.r[e] = gr[(size_t)r * 2u * a.width];
            x.i[e] = gr[(size_t)r * 2u * a.width + a.block];
            if (GATE) x.y[e] = act_load(y + (size_t)r * a.ldy);
        }
    }
    __device__ __forceinline__ void step(const Rows& x, uint32_t e, float& decay, float& add) const {
        if (sizeof(T) == 2) lru_step_fast(x.r[e] + rb, x.i[e] + ib, rate, x.u[e], decay, add);
        else lru_step(x.r[e] + rb, x.i[e] + ib, rate, x.u[e], decay, add);
    }
};

// Chunks with a successor, which are whole.
template <typename T>
__global__ __launch_bounds__(64) void lru_ends_kernel(const LruScanArgs a) {
    using Column = LruColumn<T>;
    const uint32_t c = blockIdx.x * 64u + threadIdx.x, r0 = blockIdx.y * kLruChunk;
    if (c >= a.width) return;
    const Column col(a, c);
    typename Column::Rows x[2];
    col.template fetch<false>(x[0], r0, nullptr);
    col.template fetch<false>(x[1], r0 + Column::kHalf, nullptr);
    float prod = 1.f, end = 0.f;
#pragma unroll
    for (uint32_t h = 0; h < 2; ++h)
#pragma unroll
        for (uint32_t e = 0; e < Column::kHalf; ++e) {
            float decay, add;
            col.step(x[h], e, decay, add);
            prod *= decay;
            end = fmaf(decay, end, add);
        }
    float* o = a.carry + (size_t)blockIdx.y * 2u * a.width + c;
    o[0] = prod;
    o[a.width] = end;
    // the last chunk of the next launch replaces the state while others still start from it: they read this copy
    if (blockIdx.y == 0) a.carry[(size_t)gridDim.y * 2u * a.width + c] = a.state[c];
}

template <typename T>
__global__ __launch_bounds__(64) void lru_out_kernel(const LruScanArgs a) {
    using Column = LruColumn<T>;
    const uint32_t c = blockIdx.x * 64u + threadIdx.x, chunk = blockIdx.y, r0 = chunk * kLruChunk;
    if (c >= a.width) return;
    const Column col(a, c);
    T* y = reinterpret_cast<T*>(a.y) + c;
    typename Column::Rows x[2];
    col.template fetch<true>(x[0], r0, y);
    col.template fetch<true>(x[1], r0 + Column::kHalf, y);
    const float* e = a.carry + c;
    float S = gridDim.y == 1u ? a.state[c] : e[(size_t)(gridDim.y - 1u) * 2u * a.width];
    constexpr uint32_t kPrefix = 16;   // chunks whose ends are requested together
    for (uint32_t k0 = 0; k0 < chunk; k0 += kPrefix) {
        float d[kPrefix], b[kPrefix];
#pragma unroll
        for (uint32_t i = 0; i < kPrefix; ++i) {
            const size_t k = k0 + i < chunk ? k0 + i : chunk - 1u;
            d[i] = e[k * 2u * a.width];
            b[i] = e[k * 2u * a.width + a.width];
        }
#pragma unroll
        for (uint32_t i = 0; i < kPrefix; ++i)
            if (k0 + i < chunk) S = fmaf(d[i], S, b[i]);
    }
#pragma unroll
    for (uint32_t h = 0; h < 2; ++h)
#pragma unroll
        for (uint32_t i = 0; i < Column::kHalf; ++i) {
            const uint32_t r = r0 + h * Column::kHalf + i;
            if (r < a.rows) {
                float decay, add;
                col.step(x[h], i, decay, add);
                S = fmaf(decay, S, add);
                act_store(y + (size_t)r * a.ldy, S * x[h].y[i]);
            }
        }
    if (r0 + kLruChunk >= a.rows) a.state[c] = S;
}

}  // namespace

fk_status plan_lru_scan(const LruScanArgs& a, uint32_t act, Launch* out) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, "lru scan: act must be 16 or 32");
    if (!a.u || !a.gates || !a.rb || !a.ib || !a.lam || !a.state || !a.y || !a.carry || !a.rows || !a.width || !a.block || a.width % a.block || a.ldx < a.width || a.ldy < a.width)
        return set_error(FK_ERR_INVALID, "lru scan: bad arguments");
    const uint32_t chunks = (a.rows + kLruChunk - 1) / kLruChunk, cols = (a.width + 63) / 64;
    if (chunks > 65535) return set_error(FK_ERR_UNSUPPORTED, "lru scan: too many rows");
    Launch fin;
    fin.func = act == 16 ? (const void*)&lru_out_kernel<uint16_t> : (const void*)&lru_out_kernel<float>;
    fin.grid = dim3(cols, chunks, 1);
    fin.block = dim3(64, 1, 1);
    fin.set_args(a);
    if (chunks == 1) {
        *out = fin;
        return FK_OK;
    }
    out->func = act == 16 ? (const void*)&lru_ends_kernel<uint16_t> : (const void*)&lru_ends_kernel<float>;
    out->grid = dim3(cols, chunks - 1, 1);
    out->block = dim3(64, 1, 1);
    out->shmem = 0;
    out->set_args(a);
    out->then.push_back(fin);
    return FK_OK;
}

}  // namespace fk
