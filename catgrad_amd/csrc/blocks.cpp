// Entry points of the decoder blocks (the last section of include/catgrad_hip.h): argument checks, views, the growing
// key / value cache, and which kernels a call takes.  The kernels are in block_rows.hip, block_inputs.hip, block_experts.hip,
// block_attention*.hip and block_delta.hip; products of more than a few rows go through launch_matmul like the trait's.
#include "blocks.hpp"

#include <algorithm>
#include <cmath>

namespace cg {
namespace {

// The consumed references of a block's tensor arguments, and the temporaries made from them.
struct Held {
    std::vector<cg_tensor *> t;
    ~Held() {
        for (cg_tensor *x : t) release(x);
    }
    cg_tensor *add(cg_tensor *x) {
        t.push_back(x);
        return x;
    }
};

// Pool memory for the duration of a call (stream-ordered: whoever gets it next queues behind this call's kernels).
struct Scratch {
    explicit Scratch(cg_backend *b) : be(b) {}
    ~Scratch() {
        for (auto &a : mem) be->pool.free(a.first, a.second);
    }
    int get(size_t bytes, void **p) {
        size_t cls;
        int rc = be->pool.alloc(bytes ? bytes : 4, p, &cls);
        if (!rc) mem.emplace_back(*p, cls);
        return rc;
    }
    cg_backend *be;
    std::vector<std::pair<void *, size_t>> mem;
};

int check_float(const cg_tensor *t, const char *what) {
    return is_f(t->dt) ? CG_OK : fail(CG_ERR_DTYPE, "%s: expected a floating-point tensor", what);
}

// t as rows of its last axis, `rows` x `features`, every row with unit stride and one distance from row to row.
int rows_of(cg_backend *be, Held &h, cg_tensor *t, int64_t rows, int64_t features, Rows *out, const char *what) {
    if (int rc = check_float(t, what)) return rc;
    if (t->rank < 1 || t->dims[t->rank - 1] != features || numel(t) != rows * features)
        return fail(CG_ERR_SHAPE, "%s: expected %lld rows of %lld", what, (long long)rows, (long long)features);
    if (int rc = ensure_concrete(t)) return rc;
    bool regular = !t->uniform && (features == 1 || t->strides[t->rank - 1] == 1);
    int64_t pitch = features, run = 0; // run: distance after which the next outer axis has to continue
    for (int d = t->rank - 2; d >= 0 && regular; d--) {
        if (t->dims[d] == 1) continue;
        if (run == 0) {
            pitch = t->strides[d];
            run = pitch;
        } else if (t->strides[d] != run) {
            regular = false;
        }
        run *= t->dims[d];
    }
    if (!regular) {
        cg_tensor *m = nullptr;
        if (int rc = materialize(be, t, &m)) return rc;
        h.add(m);
        t = m;
        pitch = features;
    }
    const void *p;
    if (int rc = device_ptr(t, &p)) return rc;
    out->p = static_cast<const float *>(p);
    out->pitch = pitch;
    return CG_OK;
}

// a small parameter as dense words
int dense_of(cg_backend *be, Held &h, cg_tensor *t, int64_t n, const float **out, const char *what) {
    if (int rc = check_float(t, what)) return rc;
    if (numel(t) != n) return fail(CG_ERR_SHAPE, "%s: expected %lld elements", what, (long long)n);
    if (int rc = ensure_concrete(t)) return rc;
    if (t->uniform || !is_contiguous(t)) {
        cg_tensor *m = nullptr;
        if (int rc = materialize(be, t, &m)) return rc;
        t = h.add(m);
    }
    const void *p;
    if (int rc = device_ptr(t, &p)) return rc;
    *out = static_cast<const float *>(p);
    return CG_OK;
}

// A weight matrix [n, k] (n 0: any).  `view`: the tensor as the general products take it.
int weight_of(cg_backend *be, Held &h, cg_tensor *t, int64_t k, Weight *out, cg_tensor **view, const char *what) {
    if (t->dt != CG_F32 && t->dt != CG_BF16) return fail(CG_ERR_DTYPE, "%s: weights are f32 or bf16", what);
    if (t->rank != 2 || t->dims[1] != k || t->dims[0] < 1) return fail(CG_ERR_SHAPE, "%s: incompatible weight matrix", what);
    if (int rc = ensure_concrete(t)) return rc;
    if (t->uniform || (k > 1 && t->strides[1] != 1) || (t->dims[0] > 1 && t->strides[0] < k)) {
        cg_tensor *m = nullptr;
        if (int rc = materialize(be, t, &m)) return rc;
        t = h.add(m);
    }
    int fmt;
    if (int rc = device_ptr_fmt(t, &out->p, &fmt)) return rc;
    if (fmt != kFmtWords && fmt != kFmtBF16) {
        if (int rc = device_ptr(t, &out->p)) return rc;
        fmt = kFmtWords;
    }
    out->fmt = fmt;
    out->n = (uint32_t)t->dims[0];
    out->k = (uint32_t)k;
    out->pitch = t->dims[0] > 1 ? t->strides[0] : k;
    if (view) *view = t;
    return CG_OK;
}

int check_sizes(int64_t rows, int64_t a, int64_t b) {
    return rows < (1ll << 31) && a < (1ll << 31) && b < (1ll << 31) ? CG_OK : fail(CG_ERR_UNSUPPORTED, "block: an extent exceeds 2^31");
}

// w^T and a dense f32 result as the general product takes them, on the stack; their buffers are borrowed.
struct ProductViews {
    cg_tensor wt, out;
    Buffer ybuf;
    ProductViews(cg_backend *be, const cg_tensor *w, int64_t rows, float *y) {
        const int64_t N = w->dims[0], K = w->dims[1];
        wt.be = be;
        wt.buf = w->buf;
        wt.dt = w->dt;
        wt.rank = 2;
        wt.dims[0] = K;
        wt.dims[1] = N;
        wt.strides[0] = 1;
        wt.strides[1] = N > 1 ? w->strides[0] : K;
        wt.offset = w->offset;
        ybuf.be = be;
        ybuf.ptr = y;
        ybuf.elems = rows * N;
        out.be = be;
        out.buf = &ybuf;
        out.dt = w->dt; // f32 words hold the unrounded sums
        out.rank = 2;
        out.dims[0] = rows;
        out.dims[1] = N;
        out.strides[0] = N;
        out.strides[1] = 1;
    }
    ~ProductViews() { wt.buf = out.buf = nullptr; }
};

// A left operand [rows, K] in the form that its product with these weights reads: patterns when it takes them as they lie,
// else words that hold rounded values.  *tiles: the product is for the 128-wide tiles, it does not fill the device with others.
int product_operand(cg_backend *be, int64_t rows, const Weight &weight, cg_tensor *w, cg_tensor **out, bool *tiles) {
    const int64_t K = weight.k, xd[2] = {rows, K};
    cg_tensor *x = nullptr;
    *tiles = false;
    if (w->dt == CG_BF16 && K % 8 == 0 && (rows >= 256 || takes_bf16_tiles((uint32_t)rows, weight))) {
        if (int rc = new_dense(be, CG_BF16, xd, 2, &x, 0, kFmtBF16)) return rc;
        ProductViews v(be, w, rows, nullptr);
        *tiles = rows < 256 || launch_matmul(be, x, &v.wt, nullptr) != CG_OK;
        if (*tiles && !takes_bf16_tiles((uint32_t)rows, weight)) {
            *tiles = false;
            release(x);
            x = nullptr;
        }
    }
    if (!x)
        if (int rc = new_dense(be, w->dt, xd, 2, &x)) return rc;
    *out = x;
    return CG_OK;
}
// x . w^T -> y (dense f32), x as product_operand has made it
int operand_product(cg_backend *be, cg_tensor *x, bool tiles, const Weight &weight, cg_tensor *w, float *y) {
    if (tiles) {
        const int rc = launch_bf16_tiles(be, x->buf->ptr, (uint32_t)x->dims[0], weight, y);
        if (rc != kDeclined) return rc;
    }
    ProductViews v(be, w, x->dims[0], y);
    return launch_matmul(be, x, &v.wt, &v.out);
}

// in[rows, k] . w^T -> y [rows, n] (dense f32) for any number of rows: the operand in memory in the form the weights ask
// for, then the general product.
int general_product(cg_backend *be, Held &h, const ProductInput &in, uint32_t rows, const Weight &weight, cg_tensor *w, float *y) {
    const bool bf16 = w->dt == CG_BF16;
    if (!bf16 && !in.gamma && !in.poly && !in.x2.p) { // the operand as it lies
        Buffer xbuf;
        xbuf.be = be;
        xbuf.ptr = const_cast<float *>(in.x.p);
        cg_tensor xv;
        xv.be = be;
        xv.buf = &xbuf;
        xv.dt = CG_F32;
        xv.rank = 2;
        xv.dims[0] = rows;
        xv.dims[1] = in.k;
        xv.strides[0] = in.x.pitch;
        xv.strides[1] = 1;
        const int rc = operand_product(be, &xv, false, weight, w, y);
        xv.buf = nullptr;
        drop_packed(&xbuf);
        return rc;
    }
    cg_tensor *x = nullptr;
    bool tiles = false;
    if (int rc = product_operand(be, rows, weight, w, &x, &tiles)) return rc;
    h.add(x);
    if (int rc = launch_product_input(be, in, rows, x->buf->ptr, bf16, x->buf->fmt)) return rc;
    return operand_product(be, x, tiles, weight, w, y);
}

// u32 values, one per element of t
int tokens_of(cg_backend *be, Held &h, cg_tensor *t, Tokens *out, const char *what) {
    if (t->dt != CG_U32) return fail(CG_ERR_DTYPE, "%s: expected u32 tokens", what);
    if (int rc = ensure_concrete(t)) return rc;
    if (t->uniform && numel(t) == 1) {
        out->value = t->ubits;
        return CG_OK;
    }
    if (t->uniform || !is_contiguous(t)) {
        cg_tensor *m = nullptr;
        if (int rc = materialize(be, t, &m)) return rc;
        t = h.add(m);
    }
    const void *p;
    if (int rc = device_ptr(t, &p)) return rc;
    out->p = static_cast<const uint32_t *>(p);
    return CG_OK;
}

// An embedding table [n, width], f32 or bf16.
int table_of(cg_backend *be, Held &h, cg_tensor *t, int64_t width, Table *out, const char *what) {
    Weight w;
    if (int rc = weight_of(be, h, t, width, &w, nullptr, what)) return rc;
    out->p = w.p;
    out->pitch = w.pitch;
    out->fmt = w.fmt;
    return CG_OK;
}

// Weights of any rank as one dense block, in words or bfloat16 patterns.
int dense_weights(cg_backend *be, Held &h, cg_tensor *t, const void **p, int *fmt, const char *what) {
    if (t->dt != CG_F32 && t->dt != CG_BF16) return fail(CG_ERR_DTYPE, "%s: weights are f32 or bf16", what);
    if (int rc = ensure_concrete(t)) return rc;
    if (t->uniform || !is_contiguous(t)) {
        cg_tensor *m = nullptr;
        if (int rc = materialize(be, t, &m)) return rc;
        t = h.add(m);
    }
    if (int rc = device_ptr_fmt(t, p, fmt)) return rc;
    if (*fmt != kFmtWords && *fmt != kFmtBF16) {
        *fmt = kFmtWords;
        return device_ptr(t, p);
    }
    return CG_OK;
}

// The arguments of a mixture of experts, checked.
int experts_of(cg_backend *be, Held &h, const cg_experts &e, int64_t rows, int64_t width, ExpertsPlan *p) {
    if (!e.h || !e.logits || !e.gate_up || !e.down) return fail(CG_ERR_ARG, "experts: null argument");
    if (e.gate_up->rank != 4 || e.down->rank != 3 || e.gate_up->dt != e.down->dt) return fail(CG_ERR_SHAPE, "experts: bad ranks or dtypes");
    const int64_t E = e.gate_up->dims[0], F = e.gate_up->dims[2], groups = e.groups ? (int64_t)e.groups : 1, keep = e.groups ? (int64_t)e.keep : 1;
    if (E < 1 || F < 1 || e.gate_up->dims[1] != 2 || e.gate_up->dims[3] != width || e.down->dims[0] != E || e.down->dims[1] != width || e.down->dims[2] != F)
        return fail(CG_ERR_SHAPE, "experts: incompatible weights");
    if (E % groups || keep < 1 || keep > groups || e.top < 1 || (int64_t)e.top > keep * (E / groups) || E > 65535) return fail(CG_ERR_ARG, "experts: bad counts");
    if (int rc = check_sizes(rows * (int64_t)e.top, F, width)) return rc;
    *p = {};
    p->rows = (uint32_t)rows;
    p->width = (uint32_t)width;
    p->ff = (uint32_t)F;
    p->experts = (uint32_t)E;
    p->top = (uint32_t)e.top;
    p->groups = (uint32_t)groups;
    p->keep = (uint32_t)keep;
    p->limit = e.limit;
    p->slope = e.slope;
    if (numel(e.h) != rows * width) return fail(CG_ERR_SHAPE, "experts h: expected %lld rows of %lld", (long long)rows, (long long)width);
    if (int rc = dense_weights(be, h, e.h, &p->h, &p->h_fmt, "experts h")) return rc;
    if (int rc = dense_of(be, h, e.logits, rows * E, &p->logits, "experts logits")) return rc;
    if (e.correction)
        if (int rc = dense_of(be, h, e.correction, E, &p->correction, "experts correction")) return rc;
    int f2;
    if (int rc = dense_weights(be, h, e.gate_up, &p->gate_up, &p->fmt, "experts gate_up")) return rc;
    if (int rc = dense_weights(be, h, e.down, &p->down, &f2, "experts down")) return rc;
    if (f2 != p->fmt) { // one of them small enough to lie in words: both as words
        p->fmt = kFmtWords;
        for (auto &w : {std::make_pair(e.gate_up, &p->gate_up), std::make_pair(e.down, &p->down)}) {
            cg_tensor *t = w.first;
            if (t->uniform || !is_contiguous(t)) {
                cg_tensor *m = nullptr;
                if (int rc = materialize(be, t, &m)) return rc;
                t = h.add(m);
            }
            if (int rc = device_ptr(t, w.second)) return rc;
        }
    }
    return CG_OK;
}

// The cache tensor [B, G, T, n] with room for `more` rows behind its last `keep` rows: *all is a view of keep' + more rows,
// keep' = min(T, keep), whose first keep' rows are the cache's and whose others the caller writes.  In place when the
// cache ends at the frontier of a row store with room; else its kept rows move into a new one.
int cache_room(cg_backend *be, Held &h, cg_tensor *c, int64_t keep, int64_t more, int64_t window, cg_tensor **all) {
    const int64_t B = c->dims[0], G = c->dims[1], T = c->dims[2], n = c->dims[3], kept = std::min(T, keep), need = kept + more;
    if (int rc = ensure_concrete(c)) return rc;
    RowStore *rs = c->buf && !c->uniform ? c->buf->rs : nullptr;
    bool place = false;
    int64_t row0 = 0;
    if (kept > 0 && rs && rs->R == n && rs->nblocks == B * G && c->offset % n == 0) {
        row0 = c->offset / n + (T - kept);
        place = c->strides[3] == 1 && (T == 1 || c->strides[2] == n) && (G == 1 || c->strides[1] == rs->C * n) &&
                (B == 1 || c->strides[0] == G * rs->C * n) && row0 + kept + more <= rs->C &&
                !(window > 0 && rs->C > 4 * (window + more) + 4096); // (memory of a long prompt is given back)
        for (int64_t g = 0; g < rs->nblocks && place; g++) place = rs->fill[(size_t)g] == row0 + kept;
    }
    cg_tensor *v = alloc_tensor(be);
    h.add(v);
    v->dt = CG_F32;
    v->rank = 4;
    const int64_t vd[4] = {B, G, need, n};
    memcpy(v->dims, vd, sizeof vd);
    if (place) {
        v->buf = c->buf;
        v->buf->rc.fetch_add(1);
        drop_packed(v->buf);
    } else {
        row0 = 0;
        // room for as many rows again, at least 64, at most one window (or 8192 rows)
        const int64_t C = need + std::max<int64_t>(64, std::min<int64_t>(need, window > 0 ? window : 8192));
        Buffer *b = new Buffer;
        b->be = be;
        v->buf = b;
        b->rs = new RowStore;
        b->rs->R = n;
        b->rs->C = C;
        b->rs->nblocks = B * G;
        b->rs->fill.assign((size_t)(B * G), 0);
        b->elems = B * G * C * n;
        if (int rc = be->pool.alloc((size_t)b->elems * 4, &b->ptr, &b->cls)) return rc;
    }
    const int64_t C = v->buf->rs->C;
    v->strides[3] = 1;
    v->strides[2] = n;
    v->strides[1] = C * n;
    v->strides[0] = G * C * n;
    v->offset = row0 * n;
    if (!place && kept > 0) {
        cg_tensor src, dst;
        auto part = [&](cg_tensor &p, const cg_tensor *of, int64_t first) {
            p.be = be;
            p.buf = of->buf;
            p.dt = CG_F32;
            p.rank = 4;
            memcpy(p.dims, vd, sizeof vd);
            p.dims[2] = kept;
            memcpy(p.strides, of->strides, sizeof p.strides);
            p.offset = of->offset + first * of->strides[2];
            p.uniform = of->uniform;
            p.ubits = of->ubits;
        };
        part(src, c, T - kept);
        part(dst, v, 0);
        const cg_tensor *ins[1] = {&src};
        int rc = launch_elementwise(be, kCopy, CG_F32, &dst, ins, 1);
        src.buf = dst.buf = nullptr;
        if (rc) return rc;
    }
    for (int64_t &f : v->buf->rs->fill) f = row0 + need;
    *all = v;
    return CG_OK;
}

// The last `keep` rows of `all` as a new handle.
int cache_tail(cg_backend *be, const cg_tensor *all, int64_t keep, cg_tensor **out) {
    if (keep == 0) {
        const int64_t d[4] = {all->dims[0], all->dims[1], 0, all->dims[3]};
        return new_dense(be, CG_F32, d, 4, out);
    }
    cg_tensor *v = new_view(all);
    v->offset += (all->dims[2] - keep) * all->strides[2];
    v->dims[2] = keep;
    *out = v;
    return CG_OK;
}

} // namespace
} // namespace cg

using namespace cg;

#define CG_ENTER_BLOCK(b)                                                                             \
    if (!(b)) return fail(CG_ERR_ARG, "null argument");                                               \
    if ((b)->owner_gone) return fail(CG_ERR_ARG, "backend used after cg_backend_destroy");            \
    CG_HIP(hipSetDevice((b)->device));                                                                \
    if (int flush_rc = flush_deferred(b)) return flush_rc

extern "C" {

int cg_block_linear(cg_backend *b, const cg_linear_args *a, cg_tensor **out) {
    Enter entered(b);
    if (!a) return fail(CG_ERR_ARG, "null argument");
    Held h;
    for (cg_tensor *t : {a->x, a->x2, a->gamma, a->w, a->bias}) h.add(t);
    if (!a->x || !a->w || !out || a->x->rank < 1) return fail(CG_ERR_ARG, "null argument");
    CG_ENTER_BLOCK(b);
    const int64_t k1 = a->x->dims[a->x->rank - 1], k2 = a->x2 && a->x2->rank ? a->x2->dims[a->x2->rank - 1] : 0, K = k1 + k2;
    const int64_t rows = k1 ? numel(a->x) / k1 : 0;
    if (K < 1) return fail(CG_ERR_SHAPE, "block_linear: no columns");
    if (int rc = check_sizes(rows, K, a->w->rank == 2 ? a->w->dims[0] : 0)) return rc;
    ProductInput in;
    in.k1 = (uint32_t)k1;
    in.k = (uint32_t)K;
    in.eps = a->eps;
    Weight w;
    cg_tensor *wv = nullptr;
    const float *bias = nullptr;
    if (int rc = weight_of(b, h, a->w, K, &w, &wv, "block_linear")) return rc;
    if (int rc = rows_of(b, h, a->x, rows, k1, &in.x, "block_linear x")) return rc;
    if (a->x2)
        if (int rc = rows_of(b, h, a->x2, rows, k2, &in.x2, "block_linear x2")) return rc;
    if (a->gamma)
        if (int rc = dense_of(b, h, a->gamma, K, &in.gamma, "block_linear gamma")) return rc;
    if (a->bias)
        if (int rc = dense_of(b, h, a->bias, w.n, &bias, "block_linear bias")) return rc;
    int64_t od[kMaxRank];
    memcpy(od, a->x->dims, sizeof od);
    od[a->x->rank - 1] = w.n;
    if (a->groups > 1 && (!a->gamma || a->x2 || K % (int64_t)a->groups || a->groups > 65535))
        return fail(CG_ERR_ARG, "block_linear: a norm in groups needs weights, one operand, and groups that divide it");
    cg_tensor *o = nullptr;
    if (int rc = new_dense(b, CG_F32, od, a->x->rank, &o)) return rc;
    int rc = CG_OK;
    if (rows > 0) {
        float *y = static_cast<float *>(o->buf->ptr);
        Scratch tmp(b);
        if (a->groups > 1) { // a norm over parts of the row: on its own
            ConvRowsPlan c{};
            c.B = 1;
            c.S = (uint32_t)rows;
            c.width = (uint32_t)K;
            c.groups = (uint32_t)a->groups;
            c.taps = 1;
            c.eps = a->eps;
            c.x = in.x;
            c.n = 1;
            c.out[0].gamma = in.gamma;
            void *p = nullptr;
            rc = tmp.get((size_t)rows * K * 4, &p);
            c.out[0].dst = p;
            if (!rc) rc = launch_conv_rows(b, c);
            in.x = {static_cast<const float *>(p), K};
            in.gamma = nullptr;
        }
        if (rc) {
        } else if (few_rows_slots((uint64_t)rows, (uint64_t)staged_pitch((uint32_t)K) * 4)) {
            rc = launch_few_rows_linear(b, in, (uint32_t)rows, w, bias, a->scale, y);
        } else {
            rc = general_product(b, h, in, (uint32_t)rows, w, wv, y);
            if (!rc && (bias || a->scale != 1.0f)) rc = launch_affine_rows(b, y, (uint32_t)rows, w.n, bias, a->scale);
        }
    }
    if (rc) {
        release(o);
        return rc;
    }
    *out = o;
    return CG_OK;
}

int cg_block_pair_embedding(cg_backend *b, const cg_pair_embedding_args *a, cg_tensor **out, cg_tensor **previous_out) {
    Enter entered(b);
    if (!a) return fail(CG_ERR_ARG, "null argument");
    Held h;
    for (cg_tensor *t : {a->ids, a->previous, a->table, a->pairs}) h.add(t);
    if (!a->ids || !a->previous || !a->table || !a->pairs || !out || !previous_out) return fail(CG_ERR_ARG, "null argument");
    CG_ENTER_BLOCK(b);
    if (a->ids->rank != 2 || a->previous->rank != 2 || a->table->rank != 2 || a->pairs->rank != 2) return fail(CG_ERR_SHAPE, "block_pair_embedding: bad ranks");
    const int64_t B = a->ids->dims[0], S = a->ids->dims[1], W = a->table->dims[1], V = a->table->dims[0], buckets = a->pairs->dims[0] - 1;
    if (B < 1 || S < 1 || W < 1 || V < 1 || buckets < 1 || a->previous->dims[0] != B || a->pairs->dims[1] != W)
        return fail(CG_ERR_SHAPE, "block_pair_embedding: incompatible shapes");
    if (int rc = check_sizes(B * S, std::max(W, V), buckets)) return rc;
    PairEmbeddingPlan p{};
    p.B = (uint32_t)B;
    p.S = (uint32_t)S;
    p.width = (uint32_t)W;
    p.vocab = (uint32_t)V;
    p.buckets = (uint64_t)buckets;
    p.mul_prev = a->mul_prev % p.buckets;
    p.mul_cur = a->mul_cur % p.buckets;
    p.previous_n = (uint32_t)a->previous->dims[1];
    if (int rc = tokens_of(b, h, a->ids, &p.ids, "block_pair_embedding ids")) return rc;
    if (p.previous_n)
        if (int rc = tokens_of(b, h, a->previous, &p.previous, "block_pair_embedding previous")) return rc;
    if (int rc = table_of(b, h, a->table, W, &p.table, "block_pair_embedding table")) return rc;
    if (int rc = table_of(b, h, a->pairs, W, &p.pairs, "block_pair_embedding pairs")) return rc;
    const int64_t od[3] = {B, S, W}, ld[2] = {B, 1};
    cg_tensor *o = nullptr, *l = nullptr;
    int rc = new_dense(b, CG_F32, od, 3, &o);
    if (!rc) rc = new_dense(b, CG_U32, ld, 2, &l);
    if (!rc) {
        p.out = static_cast<float *>(o->buf->ptr);
        p.previous_out = static_cast<uint32_t *>(l->buf->ptr);
        rc = launch_pair_embedding(b, p);
    }
    if (rc) {
        release(o);
        release(l);
        return rc;
    }
    *out = o;
    *previous_out = l;
    return CG_OK;
}

int cg_block_conv_linear(cg_backend *b, const cg_conv_linear_args *a, cg_tensor **y, cg_tensor **kept, cg_tensor **state_out) {
    Enter entered(b);
    if (!a) return fail(CG_ERR_ARG, "null argument");
    Held h;
    bool whole = a->x && a->state && y && kept && state_out;
    h.add(a->x);
    h.add(a->state);
    for (size_t i = 0; i < a->n && i < 2; i++)
        for (cg_tensor *t : {a->in[i].gamma, a->in[i].conv, a->in[i].w}) {
            h.add(t);
            whole = whole && t;
        }
    if (!whole || a->n < 1 || a->n > 2) return fail(CG_ERR_ARG, "block_conv_linear: bad argument");
    CG_ENTER_BLOCK(b);
    if (a->x->rank != 3 || a->in[0].conv->rank != 2) return fail(CG_ERR_SHAPE, "block_conv_linear: bad ranks");
    const int64_t B = a->x->dims[0], S = a->x->dims[1], W = a->x->dims[2], taps = a->in[0].conv->dims[1], groups = a->groups ? (int64_t)a->groups : 1, rows = B * S;
    if (B < 1 || S < 1 || W < 1 || taps < 1 || taps > kMaxTaps || W % groups || groups > 65535)
        return fail(CG_ERR_SHAPE, "block_conv_linear: bad extents (at most %u taps, groups that divide the width)", kMaxTaps);
    if (int rc = check_sizes(rows, W, 0)) return rc;
    ConvRowsPlan p{};
    p.B = (uint32_t)B;
    p.S = (uint32_t)S;
    p.width = (uint32_t)W;
    p.groups = (uint32_t)groups;
    p.taps = (uint32_t)taps;
    p.eps = a->eps;
    p.n = (int)a->n;
    if (int rc = rows_of(b, h, a->x, rows, W, &p.x, "block_conv_linear x")) return rc;
    const int64_t sd[3] = {B, taps - 1, W}, od[3] = {B, S, W};
    if (a->state->uniform && a->state->ubits == 0 && numel(a->state) == B * (taps - 1) * W) p.state = nullptr;
    else if (int rc = dense_of(b, h, a->state, B * (taps - 1) * W, &p.state, "block_conv_linear state")) return rc;
    const bool few = few_rows_slots((uint64_t)rows, (uint64_t)staged_pitch((uint32_t)W) * 4) != 0;
    struct Input {
        Weight w;
        cg_tensor *wv = nullptr, *x = nullptr; // x: the operand, in the form the product takes it
        bool tiles = false;
    } in[2];
    int rc = CG_OK;
    for (size_t i = 0; i < a->n && !rc; i++) {
        const cg_conv_input &c = a->in[i];
        if (int e = dense_of(b, h, c.gamma, W, &p.out[i].gamma, "block_conv_linear gamma")) return e;
        if (c.conv->rank != 2 || c.conv->dims[1] != taps) return fail(CG_ERR_SHAPE, "block_conv_linear: filters of different lengths");
        if (int e = dense_of(b, h, c.conv, W * taps, &p.out[i].conv, "block_conv_linear conv")) return e;
        if (int e = weight_of(b, h, c.w, W, &in[i].w, &in[i].wv, "block_conv_linear")) return e;
        if (c.keep && c.keep_bf16 && in[i].wv->dt != CG_BF16) return fail(CG_ERR_DTYPE, "block_conv_linear: rows kept in bf16 go through bf16 weights");
        const int64_t xd[2] = {rows, W};
        if (few) rc = new_dense(b, c.keep && c.keep_bf16 ? CG_BF16 : CG_F32, xd, 2, &in[i].x);
        else rc = product_operand(b, rows, in[i].w, in[i].wv, &in[i].x, &in[i].tiles);
        if (!rc && !few && c.keep && c.keep_bf16 && W % 8 == 0 && in[i].x->buf->fmt == kFmtWords) { // (who reads the kept rows takes patterns)
            release(in[i].x);
            in[i].x = nullptr;
            rc = new_dense(b, CG_BF16, xd, 2, &in[i].x, 0, kFmtBF16);
        }
        h.add(in[i].x);
        if (rc) return rc;
        if (c.keep && !c.keep_bf16 && in[i].x->dt != CG_F32) return fail(CG_ERR_DTYPE, "block_conv_linear: rows kept in f32 go through f32 weights");
        p.out[i].dst = in[i].x->buf->ptr;
        p.out[i].fmt = in[i].x->buf->fmt;
        p.out[i].round = in[i].x->dt == CG_BF16;
    }
    cg_tensor *so = nullptr, *o[2] = {nullptr, nullptr};
    rc = new_dense(b, CG_F32, sd, 3, &so);
    if (!rc) {
        p.state_out = so->buf ? static_cast<float *>(so->buf->ptr) : nullptr;
        rc = launch_conv_rows(b, p);
    }
    ProductInput pi[2];
    for (size_t i = 0; i < a->n && !rc; i++) {
        const int64_t yd[3] = {B, S, in[i].w.n};
        rc = new_dense(b, CG_F32, yd, 3, &o[i]);
        pi[i].x = {static_cast<const float *>(in[i].x->buf->ptr), W};
        pi[i].k1 = pi[i].k = (uint32_t)W;
    }
    auto dst = [&](size_t i) { return static_cast<float *>(o[i]->buf->ptr); };
    int both = kDeclined;
    if (!rc && few && a->n == 2) both = launch_few_rows_linear2(b, pi, (uint32_t)rows, {in[0].w, in[1].w}, {dst(0), dst(1)});
    if (both != kDeclined) rc = both;
    for (size_t i = 0; i < a->n && !rc && both == kDeclined; i++)
        rc = few ? launch_few_rows_linear(b, pi[i], (uint32_t)rows, in[i].w, nullptr, 1.0f, dst(i)) : operand_product(b, in[i].x, in[i].tiles, in[i].w, in[i].wv, dst(i));
    if (rc) {
        release(so);
        release(o[0]);
        release(o[1]);
        return rc;
    }
    for (size_t i = 0; i < a->n; i++) {
        y[i] = o[i];
        if (!a->in[i].keep) continue;
        cg_tensor *v = new_view(in[i].x);
        v->rank = 3;
        memcpy(v->dims, od, sizeof od);
        v->strides[2] = 1;
        v->strides[1] = W;
        v->strides[0] = S * W;
        kept[i] = v;
    }
    *state_out = so;
    return CG_OK;
}

int cg_block_token_side(cg_backend *b, const cg_token_side_args *a, cg_tensor **out) {
    Enter entered(b);
    if (!a) return fail(CG_ERR_ARG, "null argument");
    Held h;
    bool whole = out != nullptr;
    for (cg_tensor *t : {a->x, a->ids, a->table, a->gate, a->proj, a->norm}) {
        h.add(t);
        whole = whole && t;
    }
    if (!whole || a->x->rank < 1) return fail(CG_ERR_ARG, "null argument");
    CG_ENTER_BLOCK(b);
    const int64_t W = a->x->dims[a->x->rank - 1], rows = W ? numel(a->x) / W : 0;
    if (a->gate->rank != 2 || a->proj->rank != 2 || a->table->rank != 2 || rows < 1) return fail(CG_ERR_SHAPE, "block_token_side: bad ranks");
    const int64_t dim = a->gate->dims[0], cols = a->table->dims[1], vocab = a->table->dims[0];
    if (dim < 1 || a->proj->dims[0] != W || (int64_t)a->first + dim > cols || numel(a->ids) != rows) return fail(CG_ERR_SHAPE, "block_token_side: incompatible shapes");
    if (int rc = check_sizes(rows, W, std::max(cols, vocab))) return rc;
    Rows x;
    Weight gate, proj;
    cg_tensor *gv = nullptr, *pv = nullptr;
    Tokens ids;
    Table table;
    const float *norm;
    if (int rc = rows_of(b, h, a->x, rows, W, &x, "block_token_side x")) return rc;
    if (int rc = weight_of(b, h, a->gate, W, &gate, &gv, "block_token_side gate")) return rc;
    if (int rc = weight_of(b, h, a->proj, dim, &proj, &pv, "block_token_side proj")) return rc;
    if (int rc = tokens_of(b, h, a->ids, &ids, "block_token_side ids")) return rc;
    if (int rc = table_of(b, h, a->table, cols, &table, "block_token_side table")) return rc;
    if (int rc = dense_of(b, h, a->norm, W, &norm, "block_token_side norm")) return rc;
    cg_tensor *o = nullptr;
    if (int rc = new_dense(b, CG_F32, a->x->dims, a->x->rank, &o)) return rc;
    Scratch tmp(b);
    void *g = nullptr, *y = nullptr;
    int rc = tmp.get((size_t)rows * dim * 4, &g);
    if (!rc) rc = tmp.get((size_t)rows * W * 4, &y);
    auto product = [&](const Rows &in, const Weight &w, cg_tensor *wv, void *dst) {
        ProductInput p;
        p.x = in;
        p.k1 = p.k = w.k;
        if (few_rows_slots((uint64_t)rows, (uint64_t)staged_pitch(w.k) * 4)) return launch_few_rows_linear(b, p, (uint32_t)rows, w, nullptr, 1.0f, static_cast<float *>(dst));
        return general_product(b, h, p, (uint32_t)rows, w, wv, static_cast<float *>(dst));
    };
    const bool few = rows <= kFewRows;
    if (!rc && few) rc = launch_side_first(b, x, (uint32_t)rows, gate, ids, table, (uint32_t)vocab, (uint32_t)a->first, static_cast<float *>(g));
    if (!rc && !few) rc = product(x, gate, gv, g);
    if (!rc && !few) rc = launch_side_gate(b, static_cast<float *>(g), ids, table, (uint32_t)vocab, (uint32_t)a->first, (uint32_t)dim, (uint32_t)rows);
    int second = kDeclined;
    if (!rc && few)
        second = launch_side_second(b, x, static_cast<const float *>(g), (uint32_t)rows, proj, norm, a->eps, a->scale, static_cast<float *>(o->buf->ptr));
    if (second != kDeclined) rc = second;
    if (!rc && second == kDeclined) rc = product({static_cast<const float *>(g), dim}, proj, pv, y);
    if (!rc && second == kDeclined) rc = launch_side_sum(b, x, static_cast<const float *>(y), norm, (uint32_t)rows, (uint32_t)W, a->eps, a->scale, static_cast<float *>(o->buf->ptr));
    if (rc) {
        release(o);
        return rc;
    }
    *out = o;
    return CG_OK;
}

int cg_block_residual(cg_backend *b, cg_tensor *x, const cg_branch *br, size_t n, float eps, float scale, const cg_experts *experts, cg_tensor **out) {
    Enter entered(b);
    Held h;
    h.add(x);
    for (size_t i = 0; br && i < n; i++)
        for (cg_tensor *t : {br[i].y, br[i].w, br[i].gate, br[i].gate_bias, br[i].poly}) h.add(t);
    if (experts)
        for (cg_tensor *t : {experts->h, experts->logits, experts->correction, experts->gate_up, experts->down}) h.add(t);
    if (!x || !out || n > 2 || (n && !br) || x->rank < 1) return fail(CG_ERR_ARG, "block_residual: bad argument");
    CG_ENTER_BLOCK(b);
    const int64_t width = x->dims[x->rank - 1], rows = width ? numel(x) / width : 0;
    if (int rc = check_sizes(rows, width, 0)) return rc;
    ResidualBranch r[2];
    cg_tensor *wv[2] = {nullptr, nullptr};
    Rows xr;
    if (int rc = rows_of(b, h, x, rows, width, &xr, "block_residual x")) return rc;
    for (size_t i = 0; i < n; i++) {
        if (!br[i].y || !br[i].w || br[i].y->rank < 1) return fail(CG_ERR_ARG, "block_residual: null argument");
        const int64_t K = br[i].y->dims[br[i].y->rank - 1];
        if (K < 1 || br[i].w->rank != 2 || br[i].w->dims[0] != width) return fail(CG_ERR_SHAPE, "block_residual: incompatible weight matrix");
        if (int rc = check_sizes(rows, K, width)) return rc;
        r[i].in.k1 = r[i].in.k = (uint32_t)K;
        r[i].in.eps = eps;
        if (int rc = weight_of(b, h, br[i].w, K, &r[i].w, &wv[i], "block_residual")) return rc;
        if (int rc = rows_of(b, h, br[i].y, rows, K, &r[i].in.x, "block_residual y")) return rc;
        if (br[i].poly)
            if (int rc = dense_of(b, h, br[i].poly, 4, &r[i].in.poly, "block_residual poly")) return rc;
        if (br[i].gate)
            if (int rc = rows_of(b, h, br[i].gate, rows, width, &r[i].gate, "block_residual gate")) return rc;
        if (br[i].gate_bias)
            if (int rc = dense_of(b, h, br[i].gate_bias, width, &r[i].gate_bias, "block_residual gate bias")) return rc;
    }
    ExpertsPlan ep{};
    if (experts && rows > 0)
        if (int rc = experts_of(b, h, *experts, rows, width, &ep)) return rc;
    cg_tensor *o = nullptr;
    if (int rc = new_dense(b, CG_F32, x->dims, x->rank, &o)) return rc;
    int rc = CG_OK;
    if (rows > 0 && width > 0) {
        float *y = static_cast<float *>(o->buf->ptr);
        const bool plain = n == 1 && !r[0].in.poly && !r[0].gate.p && r[0].w.fmt == ep.fmt;
        if (experts && rows <= kFewRows && (n == 0 || plain)) {
            Scratch tmp(b);
            void *hidden = nullptr, *chosen = nullptr;
            rc = tmp.get((size_t)rows * ep.top * ep.ff * 4, &hidden);
            if (!rc) rc = tmp.get((size_t)rows * ep.top * 4, &chosen);
            if (!rc) rc = launch_experts_first(b, ep, static_cast<float *>(hidden), static_cast<uint32_t *>(chosen));
            if (!rc)
                rc = launch_experts_second(b, ep, static_cast<float *>(hidden), static_cast<uint32_t *>(chosen), xr, n ? r[0].in.x : Rows{}, n ? &r[0].w : nullptr, scale, y);
        } else if (!experts && scale == 1.0f && takes_few_rows_residual(r, (int)n, (uint32_t)rows)) {
            rc = launch_few_rows_residual(b, xr, r, (int)n, (uint32_t)rows, (uint32_t)width, y);
        } else {
            Scratch tmp(b);
            GatedTerm t[2];
            for (size_t i = 0; i < n && !rc; i++) {
                void *p = nullptr;
                rc = tmp.get((size_t)rows * width * 4, &p);
                if (!rc) rc = general_product(b, h, r[i].in, (uint32_t)rows, r[i].w, wv[i], static_cast<float *>(p));
                t[i].y = static_cast<const float *>(p);
                t[i].gate = r[i].gate;
                t[i].gate_bias = r[i].gate_bias;
            }
            void *p = nullptr;
            int fmt = kFmtWords;
            if (experts && !rc) {
                rc = tmp.get((size_t)rows * ep.top * width * 4, &p);
                if (!rc) rc = launch_experts(b, ep, static_cast<float *>(p), &fmt);
            }
            if (!rc) rc = launch_gated_sum(b, xr, t, (int)n, (uint32_t)rows, (uint32_t)width, y, scale, p, ep.top, fmt);
        }
    }
    if (rc) {
        release(o);
        return rc;
    }
    *out = o;
    return CG_OK;
}

int cg_block_attention(cg_backend *b, const cg_attention_args *a, cg_tensor **out, cg_tensor **k_out, cg_tensor **v_out) {
    Enter entered(b);
    if (!a) return fail(CG_ERR_ARG, "null argument");
    Held h;
    for (cg_tensor *t : {a->q, a->k, a->v, a->q_norm, a->k_norm, a->talk, a->k_cache, a->v_cache}) h.add(t);
    if (!a->q || !a->k || !a->v || !a->k_cache || !a->v_cache || !out || !k_out || !v_out) return fail(CG_ERR_ARG, "null argument");
    CG_ENTER_BLOCK(b);
    const int64_t H = (int64_t)a->heads, G = (int64_t)a->kv_heads, D = (int64_t)a->dim, V = (int64_t)a->vdim;
    if (H < 1 || G < 1 || D < 1 || V < 1 || H % G || H > 4096 || D > 65536 || V > 65536) return fail(CG_ERR_ARG, "block_attention: bad head counts or sizes");
    if (a->q->rank != 3 || a->k_cache->rank != 4 || a->v_cache->rank != 4) return fail(CG_ERR_SHAPE, "block_attention: bad ranks");
    const int64_t B = a->q->dims[0], S = a->q->dims[1], T = a->k_cache->dims[2];
    const int64_t window = (int64_t)a->window, position = (int64_t)a->position;
    if (B < 1 || S < 1) return fail(CG_ERR_SHAPE, "block_attention: no tokens");
    const int64_t kd[4] = {B, G, T, D}, vd[4] = {B, G, T, V};
    for (int i = 0; i < 4; i++)
        if (a->k_cache->dims[i] != kd[i] || a->v_cache->dims[i] != vd[i]) return fail(CG_ERR_SHAPE, "block_attention: incompatible caches");
    if (a->k_cache->dt != CG_F32 || a->v_cache->dt != CG_F32) return fail(CG_ERR_DTYPE, "block_attention: caches are f32");
    if (T > position || T < (window ? std::min(position, window - 1) : position))
        return fail(CG_ERR_SHAPE, "block_attention: the cache does not hold the visible positions");
    if (int rc = check_sizes(B * S, T + S, H * std::max(D, V))) return rc;
    AttentionPlan p{};
    p.B = (uint32_t)B;
    p.S = (uint32_t)S;
    p.heads = (uint32_t)H;
    p.kv_heads = (uint32_t)G;
    p.dim = (uint32_t)D;
    p.vdim = (uint32_t)V;
    p.window = (uint32_t)std::min<int64_t>(window, 0x7FFFFFFF);
    p.position = a->position;
    p.temp_every = a->temp_every;
    p.temp_coef = a->temp_coef;
    p.scale = a->scale;
    p.eps = a->norm_eps;
    p.bias = a->distance_bias != 0;
    if (a->rot_dims % 2 || (int64_t)a->rot_dims > D || (a->rot_dims && !(a->rot_base > 0.0))) return fail(CG_ERR_ARG, "block_attention: bad rotation");
    p.rot_dims = (uint32_t)a->rot_dims;
    p.rot_log2 = a->rot_dims ? std::log2(a->rot_base) : 0.0;
    p.unit_heads = a->unit_heads != 0;
    p.mix_scores = a->mix_scores != 0 && a->talk;
    p.zero_sink = a->zero_sink != 0;
    if (int rc = rows_of(b, h, a->q, B * S, H * D, &p.q, "block_attention q")) return rc;
    if (int rc = rows_of(b, h, a->k, B * S, G * D, &p.k, "block_attention k")) return rc;
    if (int rc = rows_of(b, h, a->v, B * S, G * V, &p.v, "block_attention v")) return rc;
    if (a->q_norm)
        if (int rc = dense_of(b, h, a->q_norm, H * D, &p.q_norm, "block_attention q_norm")) return rc;
    if (a->k_norm)
        if (int rc = dense_of(b, h, a->k_norm, G * D, &p.k_norm, "block_attention k_norm")) return rc;
    if (a->talk)
        if (int rc = dense_of(b, h, a->talk, H * H, &p.talk, "block_attention talk")) return rc;
    cg_tensor *ka = nullptr, *va = nullptr;
    const int64_t keep = window ? window - 1 : T;
    if (int rc = cache_room(b, h, a->k_cache, keep, S, window, &ka)) return rc;
    if (int rc = cache_room(b, h, a->v_cache, keep, S, window, &va)) return rc;
    p.cached = (uint32_t)(ka->dims[2] - S);
    p.keys = static_cast<float *>(ka->buf->ptr) + ka->offset;
    p.values = static_cast<float *>(va->buf->ptr) + va->offset;
    p.k_block = ka->strides[1];
    p.v_block = va->strides[1];
    const int64_t od[3] = {B, S, H * V};
    cg_tensor *o = nullptr, *ko = nullptr, *vo = nullptr;
    int rc = new_dense(b, CG_F32, od, 3, &o);
    if (!rc) {
        p.out = static_cast<float *>(o->buf->ptr);
        rc = launch_attention(b, p);
    }
    const int64_t tail = window ? std::min<int64_t>(ka->dims[2], window - 1) : ka->dims[2];
    if (!rc) rc = cache_tail(b, ka, tail, &ko);
    if (!rc) rc = cache_tail(b, va, tail, &vo);
    if (rc) {
        release(o);
        release(ko);
        release(vo);
        return rc;
    }
    *out = o;
    *k_out = ko;
    *v_out = vo;
    return CG_OK;
}

int cg_block_channel_delta(cg_backend *b, const cg_channel_delta_args *a, cg_tensor **out, cg_tensor **state_out, cg_tensor **conv_out) {
    Enter entered(b);
    if (!a) return fail(CG_ERR_ARG, "null argument");
    Held h;
    bool whole = true;
    for (cg_tensor *t : {a->q, a->k, a->v, a->conv_q, a->conv_k, a->conv_v, a->beta, a->decay, a->decay_w, a->a_log, a->dt_bias, a->gate, a->gate_w,
                         a->norm, a->state, a->conv_state}) {
        h.add(t);
        whole = whole && t;
    }
    if (!whole || !out || !state_out || !conv_out) return fail(CG_ERR_ARG, "null argument");
    CG_ENTER_BLOCK(b);
    const int64_t H = (int64_t)a->heads, G = (int64_t)a->kv_heads, D = (int64_t)a->dim, V = (int64_t)a->vdim;
    if (H < 1 || G < 1 || D < 1 || V < 1 || H % G || H > 65535 || D > 256 || V > 65536)
        return fail(CG_ERR_ARG, "block_channel_delta: bad head counts or sizes (at most 256 key channels)");
    if (a->q->rank != 3 || a->conv_q->rank != 2 || a->decay_w->rank != 2 || a->gate_w->rank != 2) return fail(CG_ERR_SHAPE, "block_channel_delta: bad ranks");
    const int64_t B = a->q->dims[0], S = a->q->dims[1], taps = a->conv_q->dims[1], kc = G * D, vc = H * V;
    if (B < 1 || S < 1 || taps < 1 || taps > 64) return fail(CG_ERR_SHAPE, "block_channel_delta: bad extents");
    if (int rc = check_sizes(B * S, 2 * kc + vc, H * D)) return rc;
    DeltaPlan p{};
    p.B = (uint32_t)B;
    p.S = (uint32_t)S;
    p.heads = (uint32_t)H;
    p.kv_heads = (uint32_t)G;
    p.dim = (uint32_t)D;
    p.vdim = (uint32_t)V;
    p.taps = (uint32_t)taps;
    p.eps = a->eps;
    p.decay_rank = (uint32_t)a->decay_w->dims[1];
    p.gate_rank = (uint32_t)a->gate_w->dims[1];
    if (p.decay_rank < 1 || p.gate_rank < 1) return fail(CG_ERR_SHAPE, "block_channel_delta: a projection of rank 0");
    if (int rc = rows_of(b, h, a->q, B * S, kc, &p.q, "block_channel_delta q")) return rc;
    if (int rc = rows_of(b, h, a->k, B * S, kc, &p.k, "block_channel_delta k")) return rc;
    if (int rc = rows_of(b, h, a->v, B * S, vc, &p.v, "block_channel_delta v")) return rc;
    if (int rc = rows_of(b, h, a->beta, B * S, H, &p.beta, "block_channel_delta beta")) return rc;
    if (int rc = rows_of(b, h, a->decay, B * S, p.decay_rank, &p.decay, "block_channel_delta decay")) return rc;
    if (int rc = rows_of(b, h, a->gate, B * S, p.gate_rank, &p.gate, "block_channel_delta gate")) return rc;
    const struct {
        cg_tensor *t;
        int64_t n;
        const float **dst;
        const char *what;
    } params[] = {{a->conv_q, kc * taps, &p.conv_q, "block_channel_delta conv_q"},
                  {a->conv_k, kc * taps, &p.conv_k, "block_channel_delta conv_k"},
                  {a->conv_v, vc * taps, &p.conv_v, "block_channel_delta conv_v"},
                  {a->decay_w, H * D * p.decay_rank, &p.decay_w, "block_channel_delta decay_w"},
                  {a->gate_w, vc * p.gate_rank, &p.gate_w, "block_channel_delta gate_w"},
                  {a->a_log, H, &p.a_log, "block_channel_delta a_log"},
                  {a->dt_bias, H * D, &p.dt_bias, "block_channel_delta dt_bias"},
                  {a->norm, V, &p.norm, "block_channel_delta norm"}};
    for (const auto &q : params)
        if (int rc = dense_of(b, h, q.t, q.n, q.dst, q.what)) return rc;
    const int64_t sd[4] = {B, H, D, V}, cd[3] = {B, taps - 1, 2 * kc + vc}, od[3] = {B, S, vc};
    auto zero = [](const cg_tensor *t) { return t->uniform && t->ubits == 0; };
    if (zero(a->state) && numel(a->state) == B * H * D * V) p.state = nullptr;
    else if (int rc = dense_of(b, h, a->state, B * H * D * V, &p.state, "block_channel_delta state")) return rc;
    if ((zero(a->conv_state) || taps == 1) && numel(a->conv_state) == cd[0] * cd[1] * cd[2]) p.conv_state = nullptr;
    else if (int rc = dense_of(b, h, a->conv_state, cd[0] * cd[1] * cd[2], &p.conv_state, "block_channel_delta conv_state")) return rc;
    cg_tensor *o = nullptr, *so = nullptr, *co = nullptr;
    int rc = new_dense(b, CG_F32, od, 3, &o);
    if (!rc) rc = new_dense(b, CG_F32, sd, 4, &so);
    if (!rc) rc = new_dense(b, CG_F32, cd, 3, &co);
    if (!rc) {
        p.out = static_cast<float *>(o->buf->ptr);
        p.state_out = static_cast<float *>(so->buf->ptr);
        p.conv_out = co->buf ? static_cast<float *>(co->buf->ptr) : nullptr;
        rc = launch_channel_delta(b, p);
    }
    if (rc) {
        release(o);
        release(so);
        release(co);
        return rc;
    }
    *out = o;
    *state_out = so;
    *conv_out = co;
    return CG_OK;
}

} // extern "C"
