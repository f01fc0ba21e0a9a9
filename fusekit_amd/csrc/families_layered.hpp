// Dispatch families of the layer-list decoder (layered.hpp).  Included by dispatcher.hip inside its anonymous
// namespace, where Dispatch, SlotRW and the slot checks live.  Slots are listed in order, optional ones in brackets
// with the parameter that announces them; `act` (16 or 32) is the width of an activation element.  Row strides are
// elements of padded rows (multiples of 64).

// Walks the slots of a dispatch: checks sizes, records the access, remembers the first error.
struct SlotCursor {
    const Dispatch& d;
    SlotRW* rw;
    size_t at = 0;
    fk_status status = FK_OK;

    void* take(uint64_t bytes, bool read, bool write) {
        const size_t s = at++;
        if (status != FK_OK) return nullptr;
        if (s >= d.args.size()) {
            status = set_error(FK_ERR_INVALID, d.kernel + ": expected more than " + std::to_string(d.args.size()) + " buffers");
            return nullptr;
        }
        if (!d.args[s].ptr || d.args[s].nbytes == 0) {
            status = set_error(FK_ERR_INVALID, d.kernel + ": buffer slot " + std::to_string(s) + " is null or empty");
            return nullptr;
        }
        status = need_bytes(d, s, (size_t)bytes);
        if (read) rw->reads.push_back((uint32_t)s);
        if (write) rw->writes.push_back((uint32_t)s);
        return d.args[s].ptr;
    }
    template <typename T = void>
    const T* in(uint64_t bytes) { return (const T*)take(bytes, true, false); }
    template <typename T = void>
    T* out(uint64_t bytes) { return (T*)take(bytes, false, true); }
    template <typename T = void>
    T* inout(uint64_t bytes) { return (T*)take(bytes, true, true); }
    fk_status end() {
        if (status == FK_OK && at != d.args.size())
            return set_error(FK_ERR_INVALID, d.kernel + ": expected " + std::to_string(at) + " buffers, got " + std::to_string(d.args.size()));
        return status;
    }
};

uint64_t act_bytes(uint32_t act) { return act == 32 ? 4 : 2; }
// Bytes from the first element of row 0 to the last valid one of row rows - 1.
uint64_t rows_bytes(uint64_t rows, uint64_t ld, uint64_t width, uint64_t elem) { return ((rows - 1) * ld + width) * elem; }

// x, [mix: has_mix], [routes, weight, index, prev: top > 0], [step: has_step], [copy: ldcopy > 0], [w1, [b1: layer_norm], h1:
// has_h1], [w2, h2: has_h2]
//   {rows, width, ld, ldcopy, act, eps, top, experts, mix_parts=1}
fk_status plan_residual_norm_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    ResidualNormArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.width = d.u("width"); a.ldx = d.u("ld", a.width); a.top = d.u("top"); a.experts = d.u("experts");
    a.eps = (float)d.param("eps", 1e-6);
    if (!a.rows || !a.width) return set_error(FK_ERR_INVALID, d.kernel + ": rows / width parameters missing");
    const uint64_t x4 = (uint64_t)a.rows * a.ldx * 4, xa = (uint64_t)a.rows * a.ldx * act_bytes(act);
    SlotCursor s{d, rw};
    a.x = s.inout<float>(x4);
    a.parts = d.u("mix_parts", 1);
    if (d.u("has_mix")) a.mix = s.in<float>(x4 * a.parts);
    if (a.top) {
        a.routes = s.in(xa * a.top);
        a.weight = s.in<float>((uint64_t)a.rows * a.top * 4);
        a.index = s.in<uint32_t>((uint64_t)a.rows * a.top * 4);
        a.prev = s.in(xa);
    }
    if (d.u("has_step")) a.step = s.in<uint16_t>((uint64_t)a.ldx * 2);
    a.ldcopy = d.u("ldcopy");
    if (a.ldcopy) a.copy = s.out(rows_bytes(a.rows, a.ldcopy, a.ldx, act_bytes(act)));
    if (d.u("has_h1")) {
        a.w1 = s.in<uint16_t>((uint64_t)a.ldx * 2);
        if (d.u("layer_norm")) a.b1 = s.in<uint16_t>((uint64_t)a.ldx * 2);
        a.h1 = s.out(xa);
    }
    if (d.u("has_h2")) { a.w2 = s.in<uint16_t>((uint64_t)a.ldx * 2); a.h2 = s.out(xa); }
    FK_TRY(s.end());
    return plan_residual_norm(a, act, l);
}

// x, [z: has_z], w, y   {rows, width, groups=1, ldx, ldz, ldy, x32, act, eps}
fk_status plan_group_norm_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    GroupNormArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.width = d.u("width"); a.groups = d.u("groups", 1); a.x32 = d.u("x32");
    a.ldx = d.u("ldx"); a.ldz = d.u("ldz"); a.ldy = d.u("ldy"); a.eps = (float)d.param("eps", 1e-6);
    if (!a.rows || !a.width || a.ldx < a.width || a.ldy < a.width) return set_error(FK_ERR_INVALID, d.kernel + ": rows / width / strides missing");
    SlotCursor s{d, rw};
    a.x = s.in(rows_bytes(a.rows, a.ldx, a.width, a.x32 ? 4 : act_bytes(act)));
    if (d.u("has_z")) a.z = s.in(rows_bytes(a.rows, a.ldz, a.width, act_bytes(act)));
    a.w = s.in<uint16_t>((uint64_t)a.width * 2);
    a.y = s.out(rows_bytes(a.rows, a.ldy, a.width, act_bytes(act)));
    FK_TRY(s.end());
    return plan_group_norm(a, act, l);
}

// x, w, [row_base: ring > 0], [bias: has_bias], y, [tail: ldt > 0]
//   {rows, n, k, ldx, ldw, ldy, batch=1, xb, wb, yb, y32, transposed, ring, row_back, act,
//    fn, fn_begin, fn_end, fn2, fn2_begin (ColumnFn), tail_begin, ldt}
fk_status plan_dense_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    DenseArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.m = d.u("rows", 1); a.n = d.u("n"); a.k = d.u("k"); a.ldx = d.u("ldx", a.k); a.ldw = d.u("ldw", a.k); a.ldy = d.u("ldy");
    a.batch = d.u("batch", 1);
    a.xb = (uint64_t)d.param("xb", 0); a.wb = (uint64_t)d.param("wb", 0); a.yb = (uint64_t)d.param("yb", 0);
    a.y32 = d.u("y32"); a.transposed = d.u("transposed"); a.ring = d.u("ring"); a.row_back = d.u("row_back");
    if (!a.m || !a.n || !a.k || !a.batch) return set_error(FK_ERR_INVALID, d.kernel + ": rows / n / k parameters missing");
    const uint64_t e = act_bytes(act), ye = a.y32 ? 4 : e;
    SlotCursor s{d, rw};
    a.x = s.in(((a.batch - 1) * a.xb + (uint64_t)((a.ring ? a.ring : a.m) - 1) * a.ldx + a.k) * e);
    a.w = s.in<uint16_t>(((a.batch - 1) * a.wb + (uint64_t)(a.n - 1) * a.ldw + a.k) * 2);
    if (a.ring) a.row_base = s.in<uint32_t>(4);
    a.out.fn = d.u("fn"); a.out.begin = d.u("fn_begin"); a.out.end = d.u("fn_end"); a.out.fn2 = d.u("fn2"); a.out.begin2 = d.u("fn2_begin");
    a.out.ldt = d.u("ldt"); a.out.tail_begin = a.out.ldt ? d.u("tail_begin") : a.n;
    if (a.out.tail_begin > a.n) return set_error(FK_ERR_INVALID, d.kernel + ": tail_begin past the columns");
    if (d.u("has_bias")) a.out.bias = s.in<uint16_t>((uint64_t)a.n * 2);
    const uint64_t rows = a.transposed ? a.n : a.m, cols = a.transposed ? a.m : a.out.tail_begin;
    if (a.ldy < cols && rows > 1) return set_error(FK_ERR_INVALID, d.kernel + ": ldy below the output width");
    a.y = s.out(((a.batch - 1) * a.yb + (rows - 1) * a.ldy + cols) * ye);
    if (a.out.ldt && a.out.tail_begin < a.n) a.out.tail = s.out<float>(rows_bytes(a.m, a.out.ldt, a.n - a.out.tail_begin, 4));
    FK_TRY(s.end());
    return plan_dense(a, act, l);
}

// tokens, table, [pairs, prev, offset: buckets > 0], x, [copy: ldcopy > 0]
//   {rows, width, vocab, ldw, ld, ldcopy, buckets, mul_prev, mul_cur, scale=1, act}
fk_status plan_embed_rows_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    EmbedRowsArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.width = d.u("width"); a.vocab = d.u("vocab"); a.ldw = d.u("ldw", a.width); a.ldx = d.u("ld", a.width); a.ldcopy = d.u("ldcopy");
    a.buckets = d.u("buckets"); a.mul_prev = d.u("mul_prev"); a.mul_cur = d.u("mul_cur"); a.scale = (float)d.param("scale", 1.0);
    if (!a.rows || !a.width || !a.vocab) return set_error(FK_ERR_INVALID, d.kernel + ": rows / width / vocab parameters missing");
    SlotCursor s{d, rw};
    a.tokens = s.in<uint32_t>((uint64_t)a.rows * 4);
    a.table = s.in<uint16_t>((uint64_t)a.vocab * a.ldw * 2);
    if (a.buckets) {
        a.pairs = s.in<uint16_t>(((uint64_t)a.buckets + 1) * a.ldw * 2);
        a.prev = s.inout<uint32_t>(4);
        a.offset = s.in<uint32_t>(4);
    }
    a.x = s.out<float>((uint64_t)a.rows * a.ldx * 4);
    if (a.ldcopy) a.copy = s.out(rows_bytes(a.rows, a.ldcopy, a.ldx, act_bytes(act)));
    FK_TRY(s.end());
    return plan_embed_rows(a, act, l);
}

// x, z, w, y   {rows, heads, dim, ld, ldx, ldz, ldy, eps, act}
fk_status plan_head_norm_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    HeadNormArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.dim = d.u("dim"); a.ld = d.u("ld", a.dim); a.eps = (float)d.param("eps", 1e-6);
    const uint32_t n = a.heads * a.ld;
    a.ldx = d.u("ldx", n); a.ldz = d.u("ldz", n); a.ldy = d.u("ldy", n);
    if (!a.rows || !n || a.ldx < n || a.ldz < n || a.ldy < n) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.x = s.in<float>(rows_bytes(a.rows, a.ldx, n, 4));
    a.z = s.in(rows_bytes(a.rows, a.ldz, n, act_bytes(act)));
    a.w = s.in<uint16_t>((uint64_t)a.ld * 2);
    a.y = s.out(rows_bytes(a.rows, a.ldy, n, act_bytes(act)));
    FK_TRY(s.end());
    return plan_head_norm(a, act, l);
}

// u, q norm, k norm, freq, offset, q, cache_k, cache_v
//   {rows, heads, kv_heads, dim, dim_ld, rot_dims, ldu, k0, q0, capacity, mag=1, eps, act}
fk_status plan_qk_store_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    QkStoreArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.kv_heads = d.u("kv_heads"); a.dim = d.u("dim"); a.dim_ld = d.u("dim_ld", a.dim); a.rot_dims = d.u("rot_dims");
    a.ldu = d.u("ldu"); a.k0 = d.u("k0"); a.q0 = d.u("q0"); a.capacity = d.u("capacity"); a.eps = (float)d.param("eps", 1e-6); a.mag = (float)d.param("mag", 1.0);
    if (!a.rows || !a.heads || !a.kv_heads || !a.dim || !a.capacity) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    const uint64_t e = act_bytes(act), nq = (uint64_t)a.heads * a.dim_ld, nk = (uint64_t)a.kv_heads * a.dim_ld;
    SlotCursor s{d, rw};
    a.u = s.in(rows_bytes(a.rows, a.ldu, std::max(a.k0 + nk, a.q0 + nq), e));
    a.wq = s.in<uint16_t>(nq * 2);
    a.wk = s.in<uint16_t>(nk * 2);
    a.freq = s.in<double>(a.rot_dims >= 2 ? (uint64_t)(a.rot_dims / 2) * 8 : 1);
    a.offset = s.in<uint32_t>(4);
    a.q = s.out(a.rows * nq * e);
    a.cache_k = s.inout(nk * a.capacity * e);
    a.cache_v = s.inout(nk * a.capacity * e);
    FK_TRY(s.end());
    return plan_qk_store(a, act, l);
}

// q, cache_k, cache_v, offset, out   {rows, heads, kv_heads, dim_ld, capacity, ldo, scale, act}
fk_status plan_gqa_rows_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    GqaRowsArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.kv_heads = d.u("kv_heads"); a.dim_ld = d.u("dim_ld"); a.capacity = d.u("capacity");
    const uint64_t e = act_bytes(act), nq = (uint64_t)a.heads * a.dim_ld, nk = (uint64_t)a.kv_heads * a.dim_ld;
    a.ldo = d.u("ldo", (uint32_t)nq); a.scale = (float)d.param("scale", 1.0);
    if (!a.rows || !nq || !nk || !a.capacity) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.q = s.in(a.rows * nq * e);
    a.cache_k = s.in(nk * a.capacity * e);
    a.cache_v = s.in(nk * a.capacity * e);
    a.offset = s.in<uint32_t>(4);
    a.out = s.out(rows_bytes(a.rows, a.ldo, nq, e));
    FK_TRY(s.end());
    return plan_gqa_rows(a, act, l);
}

// xc, dt_bias, a_log, decay, beta, qk   {rows, heads, kv_heads, dim, dim_ld, ldx, ldb, act}
fk_status plan_delta_prep_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    DeltaPrepArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.kv_heads = d.u("kv_heads"); a.dim = d.u("dim"); a.dim_ld = d.u("dim_ld", a.dim); a.ldx = d.u("ldx"); a.ldb = d.u("ldb", a.heads);
    const uint64_t nk = (uint64_t)a.kv_heads * a.dim_ld, nd = (uint64_t)a.heads * a.dim_ld;
    if (!a.rows || !nk || !nd || a.ldx < 2 * nk) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.xc = s.in(rows_bytes(a.rows, a.ldx, 2 * nk, act_bytes(act)));
    a.dt_bias = s.in<uint16_t>(nd * 2);
    a.a_log = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.decay = s.inout<float>(a.rows * nd * 4);
    a.beta = s.inout<float>(rows_bytes(a.rows, a.ldb, a.heads, 4));
    a.qk = s.out<float>(a.rows * nk * 8);
    FK_TRY(s.end());
    return plan_delta_prep(a, act, l);
}

// qk, decay, beta, v, state, o   {rows, heads, kv_heads, dim_ld, vdim_ld, state_ld, ldx, ldb, act}
fk_status plan_delta_scan_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    DeltaScanArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.kv_heads = d.u("kv_heads"); a.dim_ld = d.u("dim_ld"); a.vdim_ld = d.u("vdim_ld"); a.state_ld = d.u("state_ld");
    a.ldx = d.u("ldx"); a.ldb = d.u("ldb", a.heads);
    const uint64_t nk = (uint64_t)a.kv_heads * a.dim_ld, nd = (uint64_t)a.heads * a.dim_ld, nv = (uint64_t)a.heads * a.vdim_ld;
    if (!a.rows || !nk || !nv || !a.state_ld || a.ldx < nv) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.qk = s.in<float>(a.rows * nk * 8);
    a.decay = s.in<float>(a.rows * nd * 4);
    a.beta = s.in<float>(rows_bytes(a.rows, a.ldb, a.heads, 4));
    a.v = s.in(rows_bytes(a.rows, a.ldx, nv, act_bytes(act)));
    a.state = s.inout<float>(nv * a.state_ld * 4);
    a.o = s.out<float>(a.rows * nv * 4);
    FK_TRY(s.end());
    return plan_delta_scan(a, act, l);
}

// qk, decay, beta, v, state, o (rows in whole 64s), work   (parameters of fusekit_delta_scan, bf16)
fk_status plan_delta_chunk_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    DeltaChunkArgs a;
    memset(&a, 0, sizeof(a));
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.kv_heads = d.u("kv_heads"); a.dim_ld = d.u("dim_ld"); a.vdim_ld = d.u("vdim_ld"); a.state_ld = d.u("state_ld");
    a.ldx = d.u("ldx"); a.ldb = d.u("ldb", a.heads);
    const uint64_t nk = (uint64_t)a.kv_heads * a.dim_ld, nd = (uint64_t)a.heads * a.dim_ld, nv = (uint64_t)a.heads * a.vdim_ld;
    if (!a.rows || !nk || !nv || !a.state_ld || a.ldx < nv) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.qk = s.in<float>(a.rows * nk * 8);
    a.decay = s.in<float>(a.rows * nd * 4);
    a.beta = s.in<float>(rows_bytes(a.rows, a.ldb, a.heads, 4));
    a.v = s.in<uint16_t>(rows_bytes(a.rows, a.ldx, nv, 2));
    a.state = s.inout<float>(nv * a.state_ld * 4);
    a.o = s.out<float>((a.rows + kDeltaChunk - 1) / kDeltaChunk * kDeltaChunk * nv * 4);
    a.work = s.inout(delta_chunk_work_bytes(a.rows, a.heads, a.dim_ld, a.vdim_ld));
    FK_TRY(s.end());
    return plan_delta_chunk(a, l);
}

// u, gates, r bias, i bias, lam, state, y, carry   {rows, width, block, ldx, ldy, act}; carry holds 2 * width words per 32 rows
fk_status plan_lru_scan_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    LruScanArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.width = d.u("width"); a.block = d.u("block", a.width); a.ldx = d.u("ldx", a.width); a.ldy = d.u("ldy", a.width);
    if (!a.rows || !a.width || a.ldx < a.width || a.ldy < a.width) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    const uint64_t e = act_bytes(act), w2 = (uint64_t)a.width * 2;
    SlotCursor s{d, rw};
    a.u = s.in(rows_bytes(a.rows, a.ldx, a.width, e));
    a.gates = s.in<float>(a.rows * w2 * 4);
    a.rb = s.in<uint16_t>(w2);
    a.ib = s.in<uint16_t>(w2);
    a.lam = s.in<uint16_t>(w2);
    a.state = s.inout<float>(w2 * 2);
    a.y = s.inout(rows_bytes(a.rows, a.ldy, a.width, e));
    a.carry = s.inout<float>((a.rows + kLruChunk - 1) / kLruChunk * w2 * 4);
    FK_TRY(s.end());
    return plan_lru_scan(a, act, l);
}

// logits, correction, index, weight   {rows, outputs, top, ld}
fk_status plan_route_rows_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    RouteArgs a;
    memset(&a, 0, sizeof(a));
    a.rows = d.u("rows", 1); a.outputs = d.u("outputs"); a.top = d.u("top"); a.ldl = d.u("ld", a.outputs);
    if (!a.rows || !a.outputs || a.ldl < a.outputs) return set_error(FK_ERR_INVALID, d.kernel + ": rows / outputs parameters missing");
    SlotCursor s{d, rw};
    a.logits = s.in<float>(rows_bytes(a.rows, a.ldl, a.outputs, 4));
    a.correction = s.in<uint16_t>((uint64_t)a.outputs * 2);
    a.index = s.out<uint32_t>((uint64_t)a.rows * a.top * 4);
    a.weight = s.out<float>((uint64_t)a.rows * a.top * 4);
    FK_TRY(s.end());
    return plan_route_rows(a, l);
}

// index, perm, tiles, count   {routes, experts, tile_rows}; tiles holds 16 bytes per tile
fk_status plan_route_group_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    RouteGroupArgs a;
    memset(&a, 0, sizeof(a));
    a.routes = d.u("routes"); a.experts = d.u("experts"); a.tile_rows = d.u("tile_rows", 64);
    if (!a.routes || !a.experts || !a.tile_rows || d.args.size() != 4) return set_error(FK_ERR_INVALID, d.kernel + ": four buffers and routes / experts / tile_rows needed");
    a.max_tiles = (uint32_t)(d.args[2].nbytes / 16);
    SlotCursor s{d, rw};
    a.index = s.in<uint32_t>((uint64_t)a.routes * 4);
    a.perm = s.out<uint32_t>((uint64_t)a.routes * 4);
    a.tiles = s.out<uint32_t>(((uint64_t)a.routes / a.tile_rows + a.experts) * 16);
    a.count = s.out<uint32_t>(4);
    FK_TRY(s.end());
    return plan_route_group(a, l);
}

// x, wa, [wb: pair], index, [perm, tiles, count: grouped], y
//   {routes, experts, n, k, ldx, ldw, ldy, x_div, tile_rows, x_rows, act}
fk_status plan_experts_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    ExpertArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.routes = d.u("routes"); a.experts = d.u("experts"); a.n = d.u("n"); a.k = d.u("k"); a.ldx = d.u("ldx"); a.ldw = d.u("ldw");
    a.ldy = d.u("ldy"); a.x_div = d.u("x_div", 1); a.tile_rows = d.u("tile_rows", 64);
    if (!a.routes || !a.experts || !a.n || !a.k || !a.x_div || a.ldy < a.n) return set_error(FK_ERR_INVALID, d.kernel + ": routes / experts / n / k parameters missing");
    const uint64_t w = (uint64_t)a.experts * a.n * a.ldw * 2;
    SlotCursor s{d, rw};
    a.x = s.in((uint64_t)((a.routes - 1) / a.x_div + 1) * a.ldx * act_bytes(act));
    a.wa = s.in<uint16_t>(w);
    if (d.u("pair")) a.wb = s.in<uint16_t>(w);
    a.index = s.in<uint32_t>((uint64_t)a.routes * 4);
    if (d.u("grouped")) {
        a.perm = s.in<uint32_t>((uint64_t)a.routes * 4);
        a.max_tiles = a.routes / a.tile_rows + a.experts;
        a.tiles = s.in<uint32_t>((uint64_t)a.max_tiles * 16);
        a.count = s.in<uint32_t>(4);
    }
    a.y = s.out(rows_bytes(a.routes, a.ldy, a.n, act_bytes(act)));
    FK_TRY(s.end());
    return plan_experts(a, act, l);
}

// kv, norm, freq, cache, q, offset   {rows, rank, rank_ld, ldkv, ldc, ring, heads, hs, dim_ld, rot, rot_dims, ldq, eps, act}
fk_status plan_latent_store_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    LatentStoreArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.rank = d.u("rank"); a.rank_ld = d.u("rank_ld"); a.ldkv = d.u("ldkv"); a.ldc = d.u("ldc"); a.ring = d.u("ring");
    a.heads = d.u("heads"); a.hs = d.u("hs"); a.dim_ld = d.u("dim_ld"); a.rot = d.u("rot"); a.rot_dims = d.u("rot_dims", a.rot); a.ldq = d.u("ldq");
    a.eps = (float)d.param("eps", 1e-6);
    if (!a.rows || !a.rank || !a.heads || a.ldkv < a.rank + a.rot || a.hs < a.dim_ld + a.rot || a.ldq < a.heads * a.hs)
        return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.kv = s.in<float>(rows_bytes(a.rows, a.ldkv, a.rank + a.rot, 4));
    a.norm = s.in<uint16_t>((uint64_t)a.rank * 2);
    a.freq = s.in<double>(a.rot_dims >= 2 ? (uint64_t)(a.rot_dims / 2) * 8 : 1);
    a.cache = s.inout((uint64_t)a.ring * a.ldc * act_bytes(act));
    a.q = s.inout(rows_bytes(a.rows, a.ldq, a.heads * a.hs, act_bytes(act)));
    a.offset = s.in<uint32_t>(4);
    FK_TRY(s.end());
    return plan_latent_store(a, act, l);
}

// qa, q, cache, sink, offset, out   {rows, heads, hs, dim_ld, rot, rank, rank_ld, ldc, ldq, ring, window, scale, act}
fk_status plan_latent_attn_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    LatentAttnArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.hs = d.u("hs"); a.dim_ld = d.u("dim_ld"); a.rot = d.u("rot"); a.rank = d.u("rank"); a.rank_ld = d.u("rank_ld");
    a.ldc = d.u("ldc"); a.ldq = d.u("ldq"); a.ring = d.u("ring"); a.window = d.u("window"); a.scale = (float)d.param("scale", 1.0);
    if (!a.rows || !a.heads || !a.rank_ld || a.hs < a.dim_ld + a.rot || a.ldq < a.heads * a.hs) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    const uint64_t lat = (uint64_t)a.rows * a.heads * a.rank_ld * act_bytes(act);
    SlotCursor s{d, rw};
    a.qa = s.in(lat);
    a.q = s.in(rows_bytes(a.rows, a.ldq, a.heads * a.hs, act_bytes(act)));
    a.cache = s.in((uint64_t)a.ring * a.ldc * act_bytes(act));
    a.sink = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.offset = s.in<uint32_t>(4);
    a.out = s.out(lat);
    FK_TRY(s.end());
    return plan_latent_attn(a, act, l);
}

// u, w, [b: has_bias=1], hist, offset, y   {rows, channels, taps, ldu, ldy, ldh, linear, update, act}
fk_status plan_ssm_conv_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    SsmConvArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.channels = d.u("channels"); a.taps = d.u("taps"); a.ldu = d.u("ldu"); a.ldy = d.u("ldy"); a.ldh = d.u("ldh");
    if (!a.rows || !a.channels || !a.taps || a.ldy < a.channels || a.ldh < a.channels) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    const uint64_t e = act_bytes(act);
    SlotCursor s{d, rw};
    a.u = s.in(rows_bytes(a.rows, a.ldu, a.channels, e));
    a.w = s.in<uint16_t>((uint64_t)a.channels * a.taps * 2);
    if (d.u("has_bias", 1)) a.b = s.in<uint16_t>((uint64_t)a.channels * 2);
    a.linear = d.u("linear"); a.update = d.u("update");
    a.hist = a.update ? s.inout((uint64_t)a.taps * a.ldh * e) : const_cast<void*>(s.in((uint64_t)a.taps * a.ldh * e));
    a.offset = s.in<uint32_t>(4);
    a.y = s.out(rows_bytes(a.rows, a.ldy, a.channels, e));
    FK_TRY(s.end());
    return plan_ssm_conv(a, act, l);
}

// xbc, dt, dt_bias, a_log, d, u, offset, state, hist, y
//   {rows, heads, groups, n, p, state_ld, ldx, lddt, ldy, ldu, ldh, channels, taps, act}
fk_status plan_ssm_scan_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    SsmScanArgs a;
    memset(&a, 0, sizeof(a));
    const uint32_t act = d.u("act", 16);
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.groups = d.u("groups"); a.n = d.u("n"); a.p = d.u("p"); a.state_ld = d.u("state_ld");
    a.ldx = d.u("ldx"); a.lddt = d.u("lddt"); a.ldy = d.u("ldy"); a.ldu = d.u("ldu"); a.ldh = d.u("ldh"); a.channels = d.u("channels"); a.taps = d.u("taps");
    const uint64_t e = act_bytes(act);
    if (!a.rows || !a.heads || !a.p || a.channels != a.heads * a.p + 2 * a.groups * a.n || a.ldx < a.channels || a.lddt < a.heads || a.ldh < a.channels || a.ldy < a.heads * a.p)
        return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.xbc = s.in(rows_bytes(a.rows, a.ldx, a.channels, e));
    a.dt = s.in<float>(rows_bytes(a.rows, a.lddt, a.heads, 4));
    a.dt_bias = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.a_log = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.d = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.u = s.in(rows_bytes(a.rows, a.ldu, a.channels, e));
    a.offset = s.in<uint32_t>(4);
    a.state = s.inout<float>((uint64_t)a.heads * a.p * a.state_ld * 4);
    a.hist = s.inout((uint64_t)a.taps * a.ldh * e);
    a.y = s.out(rows_bytes(a.rows, a.ldy, a.heads * a.p, e));
    FK_TRY(s.end());
    return plan_ssm_scan(a, act, l);
}

// q, k, vt, cache, sink, offset, out
//   {rows, heads, dim_ld, rot_ld, vdim_ld, rank_ld, ldq, ldk, ldv, ldo, ldc, ring, window, scale}
fk_status plan_latent_prefill_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    LatentPrefillArgs a;
    memset(&a, 0, sizeof(a));
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.dim_ld = d.u("dim_ld"); a.rot_ld = d.u("rot_ld"); a.vdim_ld = d.u("vdim_ld");
    a.rank_ld = d.u("rank_ld"); a.ldq = d.u("ldq"); a.ldk = d.u("ldk"); a.ldv = d.u("ldv"); a.ldo = d.u("ldo"); a.ldc = d.u("ldc");
    a.ring = d.u("ring"); a.window = d.u("window"); a.scale = (float)d.param("scale", 1.0);
    if (!a.rows || !a.heads || !a.window || a.ldq < a.heads * (a.dim_ld + a.rot_ld) || a.ldk < a.heads * a.dim_ld || a.ldo < a.heads * a.vdim_ld ||
        a.ldc < a.rank_ld + a.rot_ld)
        return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.q = s.in<uint16_t>(rows_bytes(a.rows, a.ldq, a.heads * (a.dim_ld + a.rot_ld), 2));
    a.k = s.in<uint16_t>(rows_bytes((uint64_t)a.window - 1 + a.rows, a.ldk, a.heads * a.dim_ld, 2));
    a.vt = s.in<uint16_t>((uint64_t)a.heads * a.vdim_ld * a.ldv * 2);
    a.cache = s.in<uint16_t>((uint64_t)a.ring * a.ldc * 2);
    a.sink = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.offset = s.in<uint32_t>(4);
    a.out = s.out<uint16_t>(rows_bytes(a.rows, a.ldo, a.heads * a.vdim_ld, 2));
    FK_TRY(s.end());
    return plan_latent_prefill(a, l);
}

// xbc, dt, dt_bias, a_log, d, u, offset, state, hist, y, chunks, decay   (parameters of fusekit_ssm_scan, bf16)
fk_status plan_ssm_chunk_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    SsmChunkArgs a;
    memset(&a, 0, sizeof(a));
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.groups = d.u("groups"); a.n = d.u("n"); a.p = d.u("p"); a.state_ld = d.u("state_ld");
    a.ldx = d.u("ldx"); a.lddt = d.u("lddt"); a.ldy = d.u("ldy"); a.ldu = d.u("ldu"); a.ldh = d.u("ldh"); a.channels = d.u("channels"); a.taps = d.u("taps");
    if (!a.rows || !a.heads || !a.p || a.channels != a.heads * a.p + 2 * a.groups * a.n || a.ldx < a.channels || a.lddt < a.heads || a.ldh < a.channels || a.ldy < a.heads * a.p)
        return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    const uint64_t chunks = (a.rows + kSsmChunk - 1) / kSsmChunk;
    SlotCursor s{d, rw};
    a.xbc = s.in<uint16_t>(rows_bytes(a.rows, a.ldx, a.channels, 2));
    a.dt = s.in<float>(rows_bytes(a.rows, a.lddt, a.heads, 4));
    a.dt_bias = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.a_log = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.d = s.in<uint16_t>((uint64_t)a.heads * 2);
    a.u = s.in<uint16_t>(rows_bytes(a.rows, a.ldu, a.channels, 2));
    a.offset = s.in<uint32_t>(4);
    a.state = s.inout<float>((uint64_t)a.heads * a.p * a.state_ld * 4);
    a.hist = s.inout<uint16_t>((uint64_t)a.taps * a.ldh * 2);
    a.y = s.out<uint16_t>(rows_bytes(a.rows, a.ldy, a.heads * a.p, 2));
    a.chunks = s.inout<float>(chunks * a.heads * a.p * a.state_ld * 4);
    a.decay = s.inout<float>(chunks * a.heads * 4);
    FK_TRY(s.end());
    return plan_ssm_chunk(a, l);
}

// qa, q, cache, offset, [tab: rotate], part, [sink, out: combine]
//   {rows, heads, hs, dim_ld, rot, rot_dims, rank_ld, ldc, ldq, ring, window, splits, span, scale}
fk_status plan_latent_split_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    LatentSplitArgs a;
    memset(&a, 0, sizeof(a));
    a.rows = d.u("rows", 1); a.heads = d.u("heads"); a.hs = d.u("hs"); a.dim_ld = d.u("dim_ld"); a.rot = d.u("rot"); a.rot_dims = d.u("rot_dims", a.rot);
    a.rank_ld = d.u("rank_ld"); a.ldc = d.u("ldc"); a.ldq = d.u("ldq"); a.ring = d.u("ring"); a.window = d.u("window");
    a.splits = d.u("splits"); a.span = d.u("span"); a.scale = (float)d.param("scale", 1.0);
    if (!a.rows || !a.heads || !a.rank_ld || a.hs < a.dim_ld + a.rot || a.ldq < a.heads * a.hs) return set_error(FK_ERR_INVALID, d.kernel + ": shape parameters missing");
    SlotCursor s{d, rw};
    a.qa = s.in<uint16_t>((uint64_t)a.rows * a.heads * a.rank_ld * 2);
    a.q = s.in<uint16_t>(rows_bytes(a.rows, a.ldq, a.heads * a.hs, 2));
    a.cache = s.in<uint16_t>((uint64_t)a.ring * a.ldc * 2);
    a.offset = s.in<uint32_t>(4);
    if (d.u("rotate")) a.tab = s.in<float>((uint64_t)std::max(a.rot_dims, 1u) * 4);
    a.part = s.inout<float>((uint64_t)a.rows * a.splits * a.heads * (a.rank_ld + 2) * 4);
    const bool combine = d.u("combine") != 0;
    if (combine) {
        a.sink = s.in<uint16_t>((uint64_t)a.heads * 2);
        a.out = s.out<uint16_t>((uint64_t)a.rows * a.heads * a.rank_ld * 2);
    }
    FK_TRY(s.end());
    return plan_latent_split(a, combine, l);
}

// Jobs side by side; every part is announced by a parameter, slots in this order:
//   products i = 0, 1 (g<i>): g<i>_mode 0: x | 1: x, [step: g<i>_step], norm weights, [norm bias: g<i>_layer_norm], [kept row:
//     g<i>_keep] | 2: x, z, norm weights | 3: partial rows, sinks | 4: x, second row; then w, [bias: g<i>_has_bias], [y:
//     n_act > 0], [y32: n_act < n]
//     {g<i>_n, _k, _ldw, _width, _n_act, _rows_per_head, _x_head, _y_head, _groups, _splits, _heads, _eps, _fn, _fn_begin,
//      _fn_end, _fn2, _fn2_begin}
//   pair: x, gate, up, index, y                     {pair_n, _k, _ldw, _ldy, _top, _experts}
//   route: logits, correction, index, weight        {route_outputs, _top}
//   store: kv, norm, freq, offset, cache, tab            {store_rank, _rank_ld, _ldc, _ring, _rot, _rot_dims, _eps}
//   scan: u, dt, conv, conv bias, dt_bias, a_log, d, offset, state, hist, y
//                                                   {scan_heads, _groups, _n, _p, _state_ld, _ldh, _taps}
//   delta: u, a1, beta, conv, a2, dt_bias, a_log, offset, state, hist, o
//                                                   {delta_heads, _kv_heads, _dim, _dim_ld, _vdim_ld, _state_ld, _rank_ld, _ldh, _taps}
//   lru: u, conv, conv bias, gates, r bias, i bias, lam, offset, state, hist, y    {lru_width, _block, _ldh, _taps}
fk_status plan_layer_jobs_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    LayerJobsArgs a;
    memset(&a, 0, sizeof(a));
    SlotCursor s{d, rw};
    for (uint32_t i = 0; i < kMaxGemvJobs; ++i) {
        const std::string g = "g" + std::to_string(i) + "_";
        auto u = [&](const char* k, uint32_t dflt = 0) { return d.u((g + k).c_str(), dflt); };
        if (!d.has((g + "n").c_str())) continue;
        GemvJob& j = a.gemv[i];
        j.mode = u("mode"); j.n = u("n"); j.k = u("k"); j.ldw = u("ldw", j.k); j.width = u("width", j.k); j.n_act = u("n_act");
        j.rows_per_head = u("rows_per_head"); j.x_head = u("x_head"); j.y_head = u("y_head", j.rows_per_head);
        j.groups = u("groups", 1); j.splits = u("splits"); j.heads = u("heads"); j.eps = (float)d.param((g + "eps").c_str(), 1e-6);
        if (!j.n || !j.k || !j.width || j.mode > kRowJoin) return set_error(FK_ERR_INVALID, d.kernel + ": product parameters missing");
        const uint64_t nh = j.rows_per_head ? j.n / j.rows_per_head : 1;
        if (nh == 0) return set_error(FK_ERR_INVALID, d.kernel + ": rows per head");
        if (j.mode == kRowPlain) j.x = s.in(((nh - 1) * j.x_head + j.k) * 2);
        else if (j.mode == kRowNorm) {
            j.x = s.in((uint64_t)j.width * 4);
            j.vec = ((uintptr_t)j.x & 15u) == 0;
            if (u("step")) j.x2 = s.in((uint64_t)j.k * 2);
            j.nw = s.in<uint16_t>((uint64_t)j.k * 2);
            if (u("layer_norm")) j.nb = s.in<uint16_t>((uint64_t)j.k * 2);
            if (u("keep")) j.keep = s.out<uint16_t>((uint64_t)j.k * 2);
        } else if (j.mode == kRowGated) {
            j.x = s.in((uint64_t)j.width * 2);
            j.x2 = s.in((uint64_t)j.width * 2);
            j.nw = s.in<uint16_t>((uint64_t)j.width * 2);
        } else if (j.mode == kRowJoin) {
            j.x = s.in((uint64_t)j.width * 4);
            j.x2 = s.in((uint64_t)j.k);
        } else {
            j.pl = j.k + 2;
            if (j.heads != nh) return set_error(FK_ERR_INVALID, d.kernel + ": heads of the partial rows");
            j.x = s.in((uint64_t)j.splits * j.heads * j.pl * 4);
            j.nw = s.in<uint16_t>((uint64_t)j.heads * 2);
        }
        j.w = s.in<uint16_t>(((uint64_t)(j.n - 1) * j.ldw + j.k) * 2);
        j.out.fn = u("fn"); j.out.begin = u("fn_begin"); j.out.end = u("fn_end"); j.out.fn2 = u("fn2"); j.out.begin2 = u("fn2_begin");
        if (u("has_bias")) j.out.bias = s.in<uint16_t>((uint64_t)j.n * 2);
        const uint64_t outs = (nh - 1) * j.y_head + (j.rows_per_head ? j.rows_per_head : j.n);
        if (j.n_act && j.n_act < j.n && j.rows_per_head) return set_error(FK_ERR_UNSUPPORTED, d.kernel + ": per-head products have one kind of output");
        if (j.n_act) j.y = s.out((j.n_act < j.n ? j.n_act : outs) * 2);
        if (j.n_act < j.n) j.y32 = s.out<float>((j.n_act ? (uint64_t)(j.n - j.n_act) : outs) * 4);
    }
    if (d.u("pair_n")) {
        PairJob& j = a.pair;
        j.n = d.u("pair_n"); j.k = d.u("pair_k"); j.ldw = d.u("pair_ldw", j.k); j.ldy = d.u("pair_ldy", j.n); j.top = d.u("pair_top"); j.experts = d.u("pair_experts");
        if (!j.k || !j.top || !j.experts || j.ldy < j.n) return set_error(FK_ERR_INVALID, d.kernel + ": expert parameters missing");
        j.x = s.in<uint16_t>((uint64_t)j.k * 2);
        j.wa = s.in<uint16_t>((uint64_t)j.experts * j.n * j.ldw * 2);
        j.wb = s.in<uint16_t>((uint64_t)j.experts * j.n * j.ldw * 2);
        j.index = s.in<uint32_t>((uint64_t)j.top * 4);
        j.y = s.out<uint16_t>(rows_bytes(j.top, j.ldy, j.n, 2));
    }
    if (d.u("route_outputs")) {
        RouteJob& j = a.route;
        j.outputs = d.u("route_outputs"); j.top = d.u("route_top");
        j.logits = s.in<float>((uint64_t)j.outputs * 4);
        j.correction = s.in<uint16_t>((uint64_t)j.outputs * 2);
        j.index = s.out<uint32_t>((uint64_t)j.top * 4);
        j.weight = s.out<float>((uint64_t)j.top * 4);
    }
    if (d.u("store_rank")) {
        StoreJob& j = a.store;
        j.rank = d.u("store_rank"); j.rank_ld = d.u("store_rank_ld"); j.ldc = d.u("store_ldc"); j.ring = d.u("store_ring"); j.rot = d.u("store_rot");
        j.rot_dims = d.u("store_rot_dims", j.rot); j.eps = (float)d.param("store_eps", 1e-6);
        j.kv = s.in<float>((uint64_t)(j.rank + j.rot) * 4);
        j.norm = s.in<uint16_t>((uint64_t)j.rank * 2);
        j.freq = s.in<double>(j.rot_dims >= 2 ? (uint64_t)(j.rot_dims / 2) * 8 : 1);
        j.offset = s.in<uint32_t>(4);
        j.cache = s.inout<uint16_t>((uint64_t)j.ring * j.ldc * 2);
        j.tab = s.out<float>((uint64_t)std::max(j.rot_dims, 1u) * 4);
    }
    if (d.u("scan_heads")) {
        ScanJob& j = a.scan;
        j.heads = d.u("scan_heads"); j.groups = d.u("scan_groups"); j.n = d.u("scan_n"); j.p = d.u("scan_p"); j.state_ld = d.u("scan_state_ld");
        j.ldh = d.u("scan_ldh"); j.taps = d.u("scan_taps");
        const uint64_t ch = (uint64_t)j.heads * j.p + 2ull * j.groups * j.n;
        if (!j.p || !j.n || !j.taps || j.ldh < ch) return set_error(FK_ERR_INVALID, d.kernel + ": state-space parameters missing");
        j.u = s.in<uint16_t>(ch * 2);
        j.dt = s.in<float>((uint64_t)j.heads * 4);
        j.w = s.in<uint16_t>(ch * j.taps * 2);
        j.b = s.in<uint16_t>(ch * 2);
        j.dt_bias = s.in<uint16_t>((uint64_t)j.heads * 2);
        j.a_log = s.in<uint16_t>((uint64_t)j.heads * 2);
        j.d = s.in<uint16_t>((uint64_t)j.heads * 2);
        j.offset = s.in<uint32_t>(4);
        j.state = s.inout<float>((uint64_t)j.heads * j.p * j.state_ld * 4);
        j.hist = s.inout<uint16_t>((uint64_t)j.taps * j.ldh * 2);
        j.y = s.out<uint16_t>((uint64_t)j.heads * j.p * 2);
    }
    if (d.u("delta_heads")) {
        DeltaJob& j = a.delta;
        j.heads = d.u("delta_heads"); j.kv_heads = d.u("delta_kv_heads"); j.dim = d.u("delta_dim"); j.dim_ld = d.u("delta_dim_ld"); j.vdim_ld = d.u("delta_vdim_ld");
        j.state_ld = d.u("delta_state_ld"); j.rank_ld = d.u("delta_rank_ld"); j.ldh = d.u("delta_ldh"); j.taps = d.u("delta_taps");
        const uint64_t nd = (uint64_t)j.heads * j.dim_ld, nv = (uint64_t)j.heads * j.vdim_ld, ch = 2ull * j.kv_heads * j.dim_ld + nv;
        if (!j.kv_heads || !j.dim || !nd || !nv || !j.taps || j.ldh < ch) return set_error(FK_ERR_INVALID, d.kernel + ": delta rule parameters missing");
        j.u = s.in<uint16_t>(ch * 2);
        j.a1 = s.in<uint16_t>((uint64_t)j.rank_ld * 2);
        j.beta = s.in<float>((uint64_t)j.heads * 4);
        j.w = s.in<uint16_t>(ch * j.taps * 2);
        j.a2 = s.in<uint16_t>(nd * j.rank_ld * 2);
        j.dt_bias = s.in<uint16_t>(nd * 2);
        j.a_log = s.in<uint16_t>((uint64_t)j.heads * 2);
        j.offset = s.in<uint32_t>(4);
        j.state = s.inout<float>(nv * j.state_ld * 4);
        j.hist = s.inout<uint16_t>((uint64_t)j.taps * j.ldh * 2);
        j.o = s.out<float>(nv * 4);
    }
    if (d.u("lru_width")) {
        LruJob& j = a.lru;
        j.width = d.u("lru_width"); j.block = d.u("lru_block"); j.ldh = d.u("lru_ldh"); j.taps = d.u("lru_taps");
        if (!j.block || !j.taps || j.ldh < j.width) return set_error(FK_ERR_INVALID, d.kernel + ": linear recurrence parameters missing");
        const uint64_t w2 = (uint64_t)j.width * 2;
        j.u = s.in<uint16_t>(w2);
        j.w = s.in<uint16_t>(w2 * j.taps);
        j.b = s.in<uint16_t>(w2);
        j.gates = s.in<uint16_t>(w2 * 2 * j.block);
        j.rb = s.in<uint16_t>(w2);
        j.ib = s.in<uint16_t>(w2);
        j.lam = s.in<uint16_t>(w2);
        j.offset = s.in<uint32_t>(4);
        j.state = s.inout<float>(w2 * 2);
        j.hist = s.inout<uint16_t>((uint64_t)j.taps * j.ldh * 2);
        j.y = s.inout<uint16_t>(w2);
    }
    FK_TRY(s.end());
    return plan_layer_jobs(a, l);
}

// x, [mix: has_mix], [att, w: ko > 0], [expert rows, down, index, weight, h2: top > 0], [step: has_step],
// [o, z, norm weights: norm_heads > 0]
//   {n, ko, ldo, kf, top, experts, norm_heads, norm_dim, norm_ld, norm_eps}
fk_status plan_layer_out_d(const Dispatch& d, Launch* l, SlotRW* rw) {
    LayerOutArgs a;
    memset(&a, 0, sizeof(a));
    a.n = d.u("n"); a.ko = d.u("ko"); a.ldo = d.u("ldo", a.ko); a.kf = d.u("kf"); a.top = d.u("top"); a.experts = d.u("experts");
    if (!a.n || a.top > kMaxRouterTop) return set_error(FK_ERR_INVALID, d.kernel + ": n / top parameters");
    SlotCursor s{d, rw};
    a.x = s.inout<float>((uint64_t)a.n * 4);
    if (d.u("has_mix")) a.mix = s.in<float>((uint64_t)a.n * 4);
    if (a.ko) {
        a.att = s.in<uint16_t>((uint64_t)a.ko * 2);
        a.wo = s.in<uint16_t>(((uint64_t)(a.n - 1) * a.ldo + a.ko) * 2);
    }
    if (a.top) {
        a.eh = s.in<uint16_t>((uint64_t)a.top * a.kf * 2);
        a.wd = s.in<uint16_t>((uint64_t)a.experts * a.n * a.kf * 2);
        a.index = s.in<uint32_t>((uint64_t)a.top * 4);
        a.weight = s.in<float>((uint64_t)a.top * 4);
        a.h2 = s.in<uint16_t>((uint64_t)a.n * 2);
    }
    if (d.u("has_step")) a.step = s.in<uint16_t>((uint64_t)a.n * 2);
    a.heads = d.u("norm_heads"); a.hdim = d.u("norm_dim"); a.hld = d.u("norm_ld", a.hdim); a.heps = (float)d.param("norm_eps", 1e-6);
    if (a.heads) {
        const uint64_t nv = (uint64_t)a.heads * a.hld;
        a.ho = s.in<float>(nv * 4);
        a.hz = s.in<uint16_t>(nv * 2);
        a.hw = s.in<uint16_t>((uint64_t)a.hld * 2);
    }
    FK_TRY(s.end());
    return plan_layer_out(a, l);
}
