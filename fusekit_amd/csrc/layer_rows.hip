// Row kernels of the layer-list decoder around its matrix products: the residual sum with its norms, grouped (gated)
// norms, the router and the per-route expert products.  One body serves bf16 and fp32 activations.
#include "act_device.hpp"
#include "layered.hpp"

namespace fk {

namespace {

constexpr int kRowBlock = 256;

// One block per row.  Every thread owns the same elements in both passes, so x, h1 and h2 may be updated in place.
template <typename T>
__global__ __launch_bounds__(kRowBlock) void residual_norm_kernel(const ResidualNormArgs a) {
    __shared__ float red[kRowBlock / kWave + 1];
    const uint32_t r = blockIdx.x;
    float* x = a.x + (size_t)r * a.ldx;
    const float* mix = a.mix ? a.mix + (size_t)r * a.ldx : nullptr;
    const T* prev = a.prev ? reinterpret_cast<const T*>(a.prev) + (size_t)r * a.ldx : nullptr;
    const T* routes = a.routes ? reinterpret_cast<const T*>(a.routes) + (size_t)r * a.top * a.ldx : nullptr;
    T* copy = a.copy ? reinterpret_cast<T*>(a.copy) + (size_t)r * a.ldcopy : nullptr;
    float ss = 0.f, sum = 0.f;
    for (uint32_t c = threadIdx.x * 4u; c < a.ldx; c += kRowBlock * 4u) {
        float4 v = *reinterpret_cast<const float4*>(x + c);
        float4 add = make_float4(0.f, 0.f, 0.f, 0.f);
        if (mix) {
            add = *reinterpret_cast<const float4*>(mix + c);
            for (uint32_t p = 1; p < a.parts; ++p) {
                const float4 m = *reinterpret_cast<const float4*>(mix + (size_t)p * a.rows * a.ldx + c);
                add.x += m.x; add.y += m.y; add.z += m.z; add.w += m.w;
            }
        }
        if (routes) {
            float4 f = make_float4(0.f, 0.f, 0.f, 0.f);
            for (uint32_t s = 0; s < a.top; ++s) {
                const float w = a.weight[(size_t)r * a.top + s];
                const float4 e = a.index[(size_t)r * a.top + s] < a.experts ? act_load4(routes + (size_t)s * a.ldx + c) : act_load4(prev + c);
                f.x = fmaf(w, e.x, f.x); f.y = fmaf(w, e.y, f.y); f.z = fmaf(w, e.z, f.z); f.w = fmaf(w, e.w, f.w);
            }
            add.x += f.x; add.y += f.y; add.z += f.z; add.w += f.w;
        }
        v.x += add.x; v.y += add.y; v.z += add.z; v.w += add.w;
        if (a.step) {
            const float4 s = act_load4(a.step + c);
            v.x += s.x; v.y += s.y; v.z += s.z; v.w += s.w;
        }
        *reinterpret_cast<float4*>(x + c) = v;
        if (copy) act_store4(copy + c, v);
        sum += (v.x + v.y) + (v.z + v.w);
        ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
    }
    if (!a.w1 && !a.w2) return;
    if (a.b1) {   // layer norm: the padding is outside the mean of the squared deviations, and its weight and bias are zero
        const float mean = block_sum<kRowBlock>(sum, red) / (float)a.width;
        __syncthreads();
        float dev = 0.f;
        for (uint32_t c = threadIdx.x * 4u; c < a.ldx; c += kRowBlock * 4u) {
            const float4 v = *reinterpret_cast<const float4*>(x + c);
            const float d[4] = {v.x - mean, v.y - mean, v.z - mean, v.w - mean};
#pragma unroll
            for (uint32_t e = 0; e < 4; ++e)
                if (c + e < a.width) dev = fmaf(d[e], d[e], dev);
        }
        const float k = 1.0f / sqrtf(block_sum<kRowBlock>(dev, red) / (float)a.width + a.eps);
        for (uint32_t c = threadIdx.x * 4u; c < a.ldx; c += kRowBlock * 4u) {
            const float4 v = *reinterpret_cast<const float4*>(x + c), w = act_load4(a.w1 + c), b = act_load4(a.b1 + c);
            act_store4(reinterpret_cast<T*>(a.h1) + (size_t)r * a.ldx + c,
                       make_float4(fmaf((v.x - mean) * k, w.x, b.x), fmaf((v.y - mean) * k, w.y, b.y), fmaf((v.z - mean) * k, w.z, b.z), fmaf((v.w - mean) * k, w.w, b.w)));
        }
        return;
    }
    ss = block_sum<kRowBlock>(ss, red);
    const float k = 1.0f / sqrtf(ss / (float)a.width + a.eps);
    for (uint32_t c = threadIdx.x * 4u; c < a.ldx; c += kRowBlock * 4u) {
        const float4 v = *reinterpret_cast<const float4*>(x + c);
        if (a.w1) {
            const float4 w = act_load4(a.w1 + c);
            act_store4(reinterpret_cast<T*>(a.h1) + (size_t)r * a.ldx + c, make_float4(v.x * k * w.x, v.y * k * w.y, v.z * k * w.z, v.w * k * w.w));
        }
        if (a.w2) {
            const float4 w = act_load4(a.w2 + c);
            act_store4(reinterpret_cast<T*>(a.h2) + (size_t)r * a.ldx + c, make_float4(v.x * k * w.x, v.y * k * w.y, v.z * k * w.z, v.w * k * w.w));
        }
    }
}

template <typename T>
__global__ __launch_bounds__(kRowBlock) void group_norm_kernel(const GroupNormArgs a) {
    __shared__ float red[kRowBlock / kWave + 1];
    const uint32_t r = blockIdx.x, part = a.width / a.groups, c0 = blockIdx.y * part;
    const T* x = reinterpret_cast<const T*>(a.x) + (size_t)r * a.ldx;
    const float* xf = reinterpret_cast<const float*>(a.x) + (size_t)r * a.ldx;
    const T* z = a.z ? reinterpret_cast<const T*>(a.z) + (size_t)r * a.ldz : nullptr;
    auto value = [&](uint32_t c) {
        float v = a.x32 ? xf[c] : act_load(x + c);
        if (z) v *= silu(act_load(z + c));
        return v;
    };
    float ss = 0.f;
    for (uint32_t c = c0 + threadIdx.x; c < c0 + part; c += kRowBlock) {
        const float v = value(c);
        ss = fmaf(v, v, ss);
    }
    ss = block_sum<kRowBlock>(ss, red);
    const float k = 1.0f / sqrtf(ss / (float)part + a.eps);
    T* y = reinterpret_cast<T*>(a.y) + (size_t)r * a.ldy;
    for (uint32_t c = c0 + threadIdx.x; c < c0 + part; c += kRowBlock) act_store(y + c, value(c) * k * bf16_bits_to_f32(a.w[c]));
}

// One block per row.  The block of row 0 is the only one that needs the token before the pass: it reads that word, then
// leaves the pass's last token in its place.
template <typename T>
__global__ __launch_bounds__(kRowBlock) void embed_rows_kernel(const EmbedRowsArgs a) {
    const uint32_t r = blockIdx.x;
    const uint32_t raw = a.tokens[r], tok = raw < a.vocab ? raw : a.vocab - 1u;
    const uint16_t* second = nullptr;
    if (a.pairs) {
        uint32_t row = a.buckets;
        if (*a.offset + r > 0u) {
            const uint32_t before = r ? a.tokens[r - 1u] : *a.prev;
            row = (uint32_t)(((uint64_t)before * a.mul_prev + (uint64_t)tok * a.mul_cur) % a.buckets);
        }
        second = a.pairs + (size_t)row * a.ldw;
        if (r == 0) {
            __syncthreads();
            if (threadIdx.x == 0) *a.prev = a.tokens[a.rows - 1u];
        }
    }
    const uint16_t* first = a.table + (size_t)tok * a.ldw;
    for (uint32_t c = threadIdx.x * 4u; c < a.ldx; c += kRowBlock * 4u) {
        float4 v = act_load4(first + c);
        v.x *= a.scale; v.y *= a.scale; v.z *= a.scale; v.w *= a.scale;
        if (second) {
            const float4 p = act_load4(second + c);
            v.x += p.x; v.y += p.y; v.z += p.z; v.w += p.w;
        }
        *reinterpret_cast<float4*>(a.x + (size_t)r * a.ldx + c) = v;
        if (a.copy) act_store4(reinterpret_cast<T*>(a.copy) + (size_t)r * a.ldcopy + c, v);
    }
}

// A wave per (row, head).
template <typename T>
__global__ __launch_bounds__(kRowBlock) void head_norm_kernel(const HeadNormArgs a) {
    const uint32_t lane = threadIdx.x & (kWave - 1u), i = blockIdx.x * (kRowBlock / kWave) + threadIdx.x / kWave;
    if (i >= a.rows * a.heads) return;
    const uint32_t r = i / a.heads, h = i - r * a.heads;
    const float* x = a.x + (size_t)r * a.ldx + (size_t)h * a.ld;
    const T* z = reinterpret_cast<const T*>(a.z) + (size_t)r * a.ldz + (size_t)h * a.ld;
    T* y = reinterpret_cast<T*>(a.y) + (size_t)r * a.ldy + (size_t)h * a.ld;
    float ss = 0.f;
    for (uint32_t c = lane * 4u; c < a.ld; c += kWave * 4u) {
        const float4 v = *reinterpret_cast<const float4*>(x + c);
        ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
    }
    const float k = 1.0f / sqrtf(wave_sum(ss) / (float)a.dim + a.eps);
    for (uint32_t c = lane * 4u; c < a.ld; c += kWave * 4u) {
        const float4 v = *reinterpret_cast<const float4*>(x + c), w = act_load4(a.w + c), g = act_load4(z + c);
        act_store4(y + c, make_float4(v.x * k * w.x * sigmoid(g.x), v.y * k * w.y * sigmoid(g.y), v.z * k * w.z * sigmoid(g.z), v.w * k * w.w * sigmoid(g.w)));
    }
}

// One wave per token.  The scores stay in registers, lane l holding outputs l, l + 64, ...; a selection round is a
// wave maximum over (choice score, lower index first).
__global__ __launch_bounds__(kWave) void route_rows_kernel(const RouteArgs a) {
    constexpr int kPer = kMaxRouterOutputs / kWave;
    const uint32_t r = blockIdx.x, lane = threadIdx.x;
    const float* z = a.logits + (size_t)r * a.ldl;
    float s[kPer];
    float mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
        const uint32_t e = lane + (uint32_t)i * kWave;
        s[i] = e < a.outputs ? z[e] : -INFINITY;
        mx = fmaxf(mx, s[i]);
    }
    mx = wave_max(mx);
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
        s[i] = expf(s[i] - mx);   // outputs past the end: exp(-inf) = 0
        sum += s[i];
    }
    sum = wave_sum(sum);
    float choice[kPer];
#pragma unroll
    for (int i = 0; i < kPer; ++i) {
        const uint32_t e = lane + (uint32_t)i * kWave;
        s[i] = s[i] / sum;
        choice[i] = e < a.outputs ? s[i] + bf16_bits_to_f32(a.correction[e]) : -INFINITY;
    }
    float mine_w = 0.f, total = 0.f;
    uint32_t mine_i = 0;
    for (uint32_t t = 0; t < a.top; ++t) {
        float best = choice[0], bs = s[0];
        uint32_t bi = lane;
#pragma unroll
        for (int i = 1; i < kPer; ++i)
            if (choice[i] > best) { best = choice[i]; bs = s[i]; bi = lane + (uint32_t)i * kWave; }
        const float top = wave_max(best);
        uint32_t win = best == top ? bi : 0xffffffffu;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const uint32_t other = (uint32_t)__shfl_xor((int)win, o, kWave);
            win = other < win ? other : win;
        }
        if (win >= a.outputs) win = 0;   // only when every choice score is NaN or -inf
        const float w = __shfl(bs, (int)(win & (kWave - 1u)), kWave);
        if (lane == t) { mine_w = w; mine_i = win; }
        total += w;
        if ((win & (kWave - 1u)) == lane) {
#pragma unroll
            for (int i = 0; i < kPer; ++i)
                if (lane + (uint32_t)i * kWave == win) choice[i] = -INFINITY;
        }
    }
    if (lane < a.top) {
        a.index[(size_t)r * a.top + lane] = mine_i;
        a.weight[(size_t)r * a.top + lane] = mine_w / (total + 1e-20f);
    }
}

// One block: counts per expert, their prefix sums, then every route takes its place.  The order of an expert's routes
// is that of arrival; no result depends on it (every route is computed on its own).
constexpr int kGroupBlock = 1024;
__global__ __launch_bounds__(kGroupBlock) void route_group_kernel(const RouteGroupArgs a) {
    __shared__ uint32_t cnt[kMaxRouterOutputs], start[kMaxRouterOutputs];
    const uint32_t tid = threadIdx.x;
    for (uint32_t e = tid; e < a.experts; e += kGroupBlock) cnt[e] = 0;
    __syncthreads();
    for (uint32_t r = tid; r < a.routes; r += kGroupBlock) {
        const uint32_t e = a.index[r];
        if (e < a.experts) atomicAdd(&cnt[e], 1u);
    }
    __syncthreads();
    // wave 0: prefix sums of the counts and of the tiles, 64 experts at a time
    if (tid < kWave) {
        uint32_t base = 0, tbase = 0;
        for (uint32_t e0 = 0; e0 < a.experts; e0 += kWave) {
            const uint32_t e = e0 + tid, c = e < a.experts ? cnt[e] : 0u, t = (c + a.tile_rows - 1u) / a.tile_rows;
            uint32_t ic = c, it = t;
#pragma unroll
            for (int o = 1; o < kWave; o <<= 1) {
                const uint32_t uc = (uint32_t)__shfl_up((int)ic, o, kWave), ut = (uint32_t)__shfl_up((int)it, o, kWave);
                if (tid >= (uint32_t)o) { ic += uc; it += ut; }
            }
            const uint32_t s = base + ic - c, ts = tbase + it - t;
            if (e < a.experts) {
                start[e] = s;
                for (uint32_t k = 0; k < t && ts + k < a.max_tiles; ++k) {
                    uint32_t* q = a.tiles + (size_t)(ts + k) * 4u;
                    const uint32_t left = c - k * a.tile_rows;
                    q[0] = e; q[1] = s + k * a.tile_rows; q[2] = left < a.tile_rows ? left : a.tile_rows; q[3] = 0;
                }
            }
            base += (uint32_t)__shfl((int)ic, kWave - 1, kWave);
            tbase += (uint32_t)__shfl((int)it, kWave - 1, kWave);
        }
        if (tid == 0) *a.count = tbase < a.max_tiles ? tbase : a.max_tiles;
    }
    __syncthreads();
    for (uint32_t r = tid; r < a.routes; r += kGroupBlock) {
        const uint32_t e = a.index[r];
        if (e < a.experts) a.perm[atomicAdd(&start[e], 1u)] = r;
    }
}

// Route by route: a wave forms one output of one route (both dot products of a gate / up pair).
template <typename T>
__global__ __launch_bounds__(kRowBlock) void expert_rows_kernel(const ExpertArgs a) {
    const uint32_t route = blockIdx.y, lane = threadIdx.x & (kWave - 1u);
    const uint32_t n = blockIdx.x * (kRowBlock / kWave) + threadIdx.x / kWave;
    const uint32_t e = a.index[route];
    if (e >= a.experts || n >= a.n) return;   // an identity route has no matrices
    const T* x = reinterpret_cast<const T*>(a.x) + (size_t)(route / a.x_div) * a.ldx;
    const uint16_t* wa = a.wa + ((size_t)e * a.n + n) * a.ldw;
    const uint16_t* wb = a.wb ? a.wb + ((size_t)e * a.n + n) * a.ldw : nullptr;
    float sa = 0.f, sb = 0.f;
    for (uint32_t c = lane * 4u; c < a.k; c += kWave * 4u) {
        const float4 v = act_load4(x + c), w = act_load4(wa + c);
        sa = fmaf(v.x, w.x, sa); sa = fmaf(v.y, w.y, sa); sa = fmaf(v.z, w.z, sa); sa = fmaf(v.w, w.w, sa);
        if (wb) {
            const float4 u = act_load4(wb + c);
            sb = fmaf(v.x, u.x, sb); sb = fmaf(v.y, u.y, sb); sb = fmaf(v.z, u.z, sb); sb = fmaf(v.w, u.w, sb);
        }
    }
    sa = wave_sum(sa);
    if (wb) sa = silu(sa) * wave_sum(sb);
    if (lane == 0) act_store(reinterpret_cast<T*>(a.y) + (size_t)route * a.ldy + n, sa);
}

fk_status check_act(uint32_t act, const char* who) {
    if (act != 16 && act != 32) return set_error(FK_ERR_INVALID, std::string(who) + ": act must be 16 or 32");
    return FK_OK;
}

template <typename A>
void fill(Launch* l, const void* f, dim3 grid, uint32_t block, uint32_t lds, const A& a) {
    l->func = f;
    l->grid = grid;
    l->block = dim3(block, 1, 1);
    l->shmem = lds;
    l->set_args(a);
}

}  // namespace

fk_status plan_experts_grouped(const ExpertArgs& a, Launch* out);   // dense_mfma.hip

fk_status plan_residual_norm(const ResidualNormArgs& a, uint32_t act, Launch* out) {
    FK_TRY(check_act(act, "residual norm"));
    if (!a.x || !a.rows || !a.width || a.ldx % kRowPad || a.ldx < a.width) return set_error(FK_ERR_INVALID, "residual norm: bad shape");
    if (a.b1 && (!a.w1 || a.w2)) return set_error(FK_ERR_INVALID, "residual norm: a layer norm is the only norm");
    if (a.copy && (a.ldcopy % 4 || a.ldcopy < a.ldx)) return set_error(FK_ERR_INVALID, "residual norm: copies go to padded rows");
    if ((a.w1 && !a.h1) || (a.w2 && !a.h2)) return set_error(FK_ERR_INVALID, "residual norm: a norm without an output");
    if (a.routes && (!a.weight || !a.index || !a.prev || !a.top)) return set_error(FK_ERR_INVALID, "residual norm: incomplete routes");
    fill(out, act == 16 ? (const void*)&residual_norm_kernel<uint16_t> : (const void*)&residual_norm_kernel<float>, dim3(a.rows), kRowBlock, 0, a);
    return FK_OK;
}

fk_status plan_group_norm(const GroupNormArgs& a, uint32_t act, Launch* out) {
    FK_TRY(check_act(act, "group norm"));
    if (!a.x || !a.w || !a.y || !a.rows || !a.groups || a.width % a.groups || !a.width) return set_error(FK_ERR_INVALID, "group norm: bad shape");
    if (a.groups > 65535) return set_error(FK_ERR_UNSUPPORTED, "group norm: too many groups");
    fill(out, act == 16 ? (const void*)&group_norm_kernel<uint16_t> : (const void*)&group_norm_kernel<float>, dim3(a.rows, a.groups), kRowBlock, 0, a);
    return FK_OK;
}

fk_status plan_embed_rows(const EmbedRowsArgs& a, uint32_t act, Launch* out) {
    FK_TRY(check_act(act, "embedding rows"));
    if (!a.tokens || !a.table || !a.x || !a.rows || !a.vocab || a.ldx % kRowPad || a.ldx < a.width || a.ldw % 4 || a.ldw < a.ldx)
        return set_error(FK_ERR_INVALID, "embedding rows: bad shape");
    if (a.pairs && (!a.buckets || !a.prev || !a.offset)) return set_error(FK_ERR_INVALID, "embedding rows: incomplete second table");
    if (a.copy && (a.ldcopy % 4 || a.ldcopy < a.ldx)) return set_error(FK_ERR_INVALID, "embedding rows: copies go to padded rows");
    fill(out, act == 16 ? (const void*)&embed_rows_kernel<uint16_t> : (const void*)&embed_rows_kernel<float>, dim3(a.rows), kRowBlock, 0, a);
    return FK_OK;
}

fk_status plan_head_norm(const HeadNormArgs& a, uint32_t act, Launch* out) {
    FK_TRY(check_act(act, "head norm"));
    if (!a.x || !a.z || !a.w || !a.y || !a.rows || !a.heads || !a.dim || a.ld < a.dim || a.ld % 4 || a.ldx % 4 || a.ldz % 4 || a.ldy % 4)
        return set_error(FK_ERR_INVALID, "head norm: bad shape");
    fill(out, act == 16 ? (const void*)&head_norm_kernel<uint16_t> : (const void*)&head_norm_kernel<float>,
         dim3((uint32_t)(((uint64_t)a.rows * a.heads + 3u) / 4u)), kRowBlock, 0, a);
    return FK_OK;
}

fk_status plan_route_rows(const RouteArgs& a, Launch* out) {
    if (!a.logits || !a.correction || !a.index || !a.weight || !a.rows) return set_error(FK_ERR_INVALID, "router: null pointer");
    if (!a.top || a.top > a.outputs) return set_error(FK_ERR_INVALID, "router: top outside 1 .. outputs");
    if (a.outputs > kMaxRouterOutputs || a.top > kMaxRouterTop) return set_error(FK_ERR_UNSUPPORTED, "router: at most 1024 outputs and top 64");
    fill(out, (const void*)&route_rows_kernel, dim3(a.rows), kWave, 0, a);
    return FK_OK;
}

fk_status plan_route_group(const RouteGroupArgs& a, Launch* out) {
    if (!a.index || !a.perm || !a.tiles || !a.count || !a.routes || !a.tile_rows) return set_error(FK_ERR_INVALID, "route group: bad arguments");
    if (a.experts > kMaxRouterOutputs) return set_error(FK_ERR_UNSUPPORTED, "route group: at most 1024 experts");
    if (a.max_tiles < a.routes / a.tile_rows + a.experts) return set_error(FK_ERR_INVALID, "route group: tile table too small");
    fill(out, (const void*)&route_group_kernel, dim3(1), kGroupBlock, 0, a);
    return FK_OK;
}

fk_status plan_experts(const ExpertArgs& a, uint32_t act, Launch* out) {
    FK_TRY(check_act(act, "experts"));
    if (!a.x || !a.wa || !a.index || !a.y || !a.routes || !a.experts || !a.n || !a.x_div) return set_error(FK_ERR_INVALID, "experts: bad arguments");
    if (a.k % kRowPad || a.k > a.ldx || a.k > a.ldw) return set_error(FK_ERR_INVALID, "experts: k must be padded and within the rows");
    if (a.perm) {
        if (act != 16) return set_error(FK_ERR_UNSUPPORTED, "experts: the grouped form takes bf16 activations");
        return plan_experts_grouped(a, out);
    }
    if (a.routes > 65535) return set_error(FK_ERR_UNSUPPORTED, "experts: at most 65535 routes route by route");
    fill(out, act == 16 ? (const void*)&expert_rows_kernel<uint16_t> : (const void*)&expert_rows_kernel<float>,
         dim3((a.n + 3u) / 4u, a.routes), kRowBlock, 0, a);
    return FK_OK;
}

}  // namespace fk
