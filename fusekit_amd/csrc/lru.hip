// Real-gated linear recurrent unit: per channel
//     S <- a S + sqrt(1 - a^2) i u,   log a = -8 r softplus(lam),   r, i = sigmoid(block-diagonal products)
// and the output S times the gate branch.  A channel is independent of all others and its recurrence is linear, so a pass
// runs in chunks of 32 tokens side by side: every chunk's product of decays and its end from a zero state, then every
// chunk once more from the state its predecessors leave, which each thread forms from their ends.
#include "lru_device.hpp"

namespace fk {

namespace {

constexpr uint32_t kLruAhead = 8;

template <typename T>
struct LruColumn {
    const LruScanArgs& a;
    const T* u;
    const float* gr;
    float rb, ib, rate;

    __device__ LruColumn(const LruScanArgs& args, uint32_t c)
        : a(args), u(reinterpret_cast<const T*>(args.u) + c), gr(args.gates + (size_t)(c / args.block) * 2u * args.block + c % args.block),
          rb(bf16_bits_to_f32(args.rb[c])), ib(bf16_bits_to_f32(args.ib[c])), rate(lru_rate(args.lam[c])) {}

    // f(row, decay, addend) for rows r0 .. r1 - 1 in order, the inputs a few rows ahead
    template <typename F>
    __device__ __forceinline__ void walk(uint32_t r0, uint32_t r1, const F& f) const {
        float uv[kLruAhead], rv[kLruAhead], iv[kLruAhead];
        auto fetch = [&](uint32_t e, uint32_t r) __attribute__((always_inline)) {
            r = r < r1 ? r : r1 - 1u;
            uv[e] = act_load(u + (size_t)r * a.ldx);
            rv[e] = gr[(size_t)r * 2u * a.width];
            iv[e] = gr[(size_t)r * 2u * a.width + a.block];
        };
#pragma unroll
        for (uint32_t e = 0; e < kLruAhead; ++e) fetch(e, r0 + e);
        for (uint32_t r = r0; r < r1; r += kLruAhead) {
#pragma unroll
            for (uint32_t e = 0; e < kLruAhead; ++e) {
                if (r + e < r1) {
                    float decay, add;
                    if (sizeof(T) == 2) lru_step_fast(rv[e] + rb, iv[e] + ib, rate, uv[e], decay, add);
                    else lru_step(rv[e] + rb, iv[e] + ib, rate, uv[e], decay, add);
                    f(r + e, decay, add);
                }
                fetch(e, r + e + kLruAhead);
            }
        }
    }
};

template <typename T>
__global__ __launch_bounds__(64) void lru_ends_kernel(const LruScanArgs a) {
    const uint32_t c = blockIdx.x * 64u + threadIdx.x, r0 = blockIdx.y * kLruChunk;
    if (c >= a.width) return;
    const LruColumn<T> col(a, c);
    float prod = 1.f, end = 0.f;
    col.walk(r0, r0 + kLruChunk, [&](uint32_t, float decay, float add) __attribute__((always_inline)) {   // the last chunk has no successor: whole chunks only
        prod *= decay;
        end = fmaf(decay, end, add);
    });
    float* o = a.carry + (size_t)blockIdx.y * 2u * a.width + c;
    o[0] = prod;
    o[a.width] = end;
}

template <typename T>
__global__ __launch_bounds__(64) void lru_out_kernel(const LruScanArgs a) {
    const uint32_t c = blockIdx.x * 64u + threadIdx.x, chunk = blockIdx.y, r0 = chunk * kLruChunk;
    if (c >= a.width) return;
    const uint32_t r1 = r0 + kLruChunk < a.rows ? r0 + kLruChunk : a.rows;
    const LruColumn<T> col(a, c);
    float S = a.state[c];
    const float* e = a.carry + c;
#pragma unroll 4
    for (uint32_t k = 0; k < chunk; ++k) S = fmaf(e[(size_t)k * 2u * a.width], S, e[(size_t)k * 2u * a.width + a.width]);
    T* y = reinterpret_cast<T*>(a.y) + c;
    col.walk(r0, r1, [&](uint32_t r, float decay, float add) __attribute__((always_inline)) {
        S = fmaf(decay, S, add);
        T* p = y + (size_t)r * a.ldy;
        act_store(p, S * act_load(p));
    });
    if (r1 != a.rows) return;
    if (gridDim.y == 1u) a.state[c] = S;
    else a.carry[(size_t)chunk * 2u * a.width + c] = S;   // other chunks still read the state: a launch of its own replaces it
}

__global__ __launch_bounds__(256) void lru_state_kernel(const LruScanArgs a) {
    const uint32_t c = blockIdx.x * 256u + threadIdx.x, chunk = (a.rows - 1u) / kLruChunk;
    if (c < a.width) a.state[c] = a.carry[(size_t)chunk * 2u * a.width + c];
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
    Launch st;
    st.func = (const void*)&lru_state_kernel;
    st.grid = dim3((a.width + 255) / 256, 1, 1);
    st.block = dim3(256, 1, 1);
    st.set_args(a);
    out->then.push_back(fin);
    out->then.push_back(st);
    return FK_OK;
}

}  // namespace fk
