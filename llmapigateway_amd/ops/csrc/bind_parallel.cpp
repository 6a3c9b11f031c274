// Bindings of the dynamic-tanh rows, attention over key and value pages,
// recurrences with a decay per channel, and experts (the rest of the hybrid
// kernels: ext_hybrid.cpp). Shapes, strides and dtypes are checked here.

#include "bind_shared.h"
#include "bind_checks.h"

extern "C" {
hipError_t launch_stream_tanh(void*, int64_t, float*, const void*, int, const void*, const void*, const int*, const float*, int, const float*, const float*, float, const float*, const float*, float, int, int, int, int, int, hipStream_t);
hipError_t launch_embed_tanh(float*, void*, int64_t, const int64_t*, const void*, const float*, const float*, float, int, int, int, int, hipStream_t);
hipError_t launch_token_shift(void*, const void*, const float*, int, void*, const int64_t*, const int*, const int*, const int*, int, int, int, int, int, hipStream_t);
hipError_t launch_head_norm(void*, int64_t, const void*, const void*, int64_t, const float*, float, int, int, int, int, int, hipStream_t);
hipError_t launch_gated_norm(void*, int64_t, const void*, const void*, int64_t, const float*, float, int, int, int, int, int, int, hipStream_t);
hipError_t launch_page_write(void*, void*, const void*, int64_t, const void*, int64_t, const int64_t*, int, int, int, int, int, hipStream_t);
hipError_t launch_clamped_glu(void*, const void*, float, int, int, int, int, hipStream_t);
hipError_t launch_soft_cap(float*, float, size_t, hipStream_t);
hipError_t launch_paged_rows(void*, int64_t, const void*, int64_t, const void*, const void*, const float*, const void*, int64_t, float, float, float, const int64_t*, const int*, const int*, const int*, int, int, int, int, int, int, int, int, float*, float*, int, hipStream_t);
hipError_t launch_paged_tiles(void*, int64_t, const void*, int64_t, const void*, const void*, const float*, const void*, int64_t, float, float, float, const int64_t*, const int*, int, int, int, int, int, int, const int*, const int*, const int*, int, int, hipStream_t);
hipError_t launch_decay_logs(float*, const void*, int64_t, const void*, const float*, const float*, int, float, int, int, int, int, int, hipStream_t);
hipError_t launch_decay_scan(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, const float*, const float*, float, int, int, int, int, float*, const int64_t*, const int*, const int*, const int*, int, int, hipStream_t);
hipError_t launch_decay_chunked(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, float*, const float*, float, int, int, int, int, float*, const int64_t*, const int*, const int*, const int*, const int*, const int*, const int*, int, int, void*, hipStream_t);
hipError_t launch_route_topk(int*, float*, const float*, const float*, float, int, int, int, hipStream_t);
hipError_t launch_route_plan(int*, int*, int*, const int*, int, int, int, int, int, hipStream_t);
hipError_t launch_expert_product(void*, int64_t, const void*, int64_t, const void*, const int*, const int*, int, int, int, float, int, int, int, int, int, int, hipStream_t);
}

namespace {

// x (fp32 stream) += or = post(d); out = norm(x), or x without a norm. d is
// delta or the experts' sum (rows, slot, weights, shared).
void stream_tanh(Tensor out, Tensor x, OptTensor delta, OptTensor rows, OptTensor slot,
                 OptTensor weights, OptTensor shared, OptTensor post_w, OptTensor post_b,
                 double post_alpha, OptTensor norm_w, OptTensor norm_b, double norm_alpha,
                 bool replace) {
    const bool f32 = is_f32(out, "out");
    TORCH_CHECK(x.dim() == 2);
    const int64_t T = x.size(0), W = x.size(1);
    f32_ptr(x, T * W, "x");
    check_rows(out, T, W, "out");
    bool v = vec8({&x, &out}, {W}), d32 = false;
    const void *dp = nullptr, *rp = nullptr, *sp = nullptr;
    const int* ip = nullptr;
    const float* wp = nullptr;
    int64_t top = 0;
    if (has(slot)) {
        TORCH_CHECK(has(rows) && has(weights) && !has(delta) && slot->dim() == 2);
        same_type(*rows, out, "rows");
        check_rows(*rows, rows->size(0), W, "rows");
        TORCH_CHECK(rows->is_contiguous());
        top = slot->size(1);
        ip = i32_ptr(*slot, T * top, "slot");
        wp = f32_ptr(*weights, T * top, "weights");
        rp = rows->data_ptr();
        v = v && vec8({&*rows}, {});
        if (has(shared)) {
            same_type(*shared, out, "shared");
            check_rows(*shared, T, W, "shared");
            TORCH_CHECK(shared->is_contiguous());
            sp = shared->data_ptr();
            v = v && vec8({&*shared}, {});
        }
    } else if (has(delta)) {
        check_rows(*delta, T, W, "delta");
        TORCH_CHECK(delta->is_contiguous());
        d32 = is_f32(*delta, "delta");
        TORCH_CHECK(d32 || !f32, "delta: bf16 beside fp32");
        dp = delta->data_ptr();
        v = v && vec8({&*delta}, {});
    }
    TORCH_CHECK(!replace || dp || ip, "replace needs delta");
    auto vec_ptr = [&](const OptTensor& t, const char* name) -> const float* {
        if (!has(t)) return nullptr;
        v = v && vec8({&*t}, {});
        return f32_ptr(*t, W, name);
    };
    const float *pw = vec_ptr(post_w, "post.w"), *pb = vec_ptr(post_b, "post.b");
    const float *nw = vec_ptr(norm_w, "norm.w"), *nb = vec_ptr(norm_b, "norm.b");
    TORCH_CHECK(!pw == !pb && !nw == !nb);
    CHECK_HIP(launch_stream_tanh(out.data_ptr(), out.stride(0), x.data_ptr<float>(), dp, d32,
                                 rp, sp, ip, wp, top, pw, pb, (float)post_alpha, nw, nb,
                                 (float)norm_alpha, replace, T, W, f32, v, current_stream()));
}

void embed_tanh(Tensor x, OptTensor x0, Tensor tokens, Tensor embed, Tensor w, Tensor b,
                double alpha) {
    const bool f32 = is_f32(embed, "embed");
    TORCH_CHECK(embed.dim() == 2 && embed.is_contiguous());
    const int64_t W = embed.size(1), T = tokens.numel();
    f32_ptr(x, T * W, "x");
    bool v = vec8({&x, &embed, &w, &b}, {W});
    if (has(x0)) {
        same_type(*x0, embed, "x0");
        check_rows(*x0, T, W, "x0");
        v = v && vec8({&*x0}, {});
    }
    CHECK_HIP(launch_embed_tanh(x.data_ptr<float>(), has(x0) ? x0->data_ptr() : nullptr,
                                has(x0) ? x0->stride(0) : 0, i64_ptr(tokens, T, "tokens"),
                                embed.data_ptr(), f32_ptr(w, W, "w"), f32_ptr(b, W, "b"),
                                (float)alpha, T, W, f32, v, current_stream()));
}

void token_shift(Tensor out, Tensor h, Tensor mu, Tensor prev, Tensor positions, Tensor cu,
                 Tensor slots, Tensor row_seg) {
    const bool f32 = is_f32(h, "h");
    same_type(h, out, "out");
    same_type(h, prev, "prev");
    TORCH_CHECK(h.dim() == 2 && h.is_contiguous() && mu.dim() == 2);
    const int64_t T = h.size(0), W = h.size(1), M = mu.size(0), S = slots.numel();
    TORCH_CHECK(out.is_contiguous() && out.numel() == M * T * W);
    TORCH_CHECK(prev.dim() == 2 && prev.is_contiguous() && prev.size(1) == W);
    CHECK_HIP(launch_token_shift(
        out.data_ptr(), h.data_ptr(), f32_ptr(mu, M * W, "mu"), M, prev.data_ptr(),
        i64_ptr(positions, T, "positions"), i32_ptr(cu, S + 1, "cu"), i32_ptr(slots, S, "slots"),
        i32_ptr(row_seg, T, "row_seg"), T, S, W, f32, vec8({&h, &out, &mu, &prev}, {W}),
        current_stream()));
}

// out = rms(y) per head * w * silu(gate)
void head_norm_gate(Tensor out, Tensor y, Tensor gate, Tensor w, int64_t heads, double eps,
                    bool sigmoid) {
    const bool f32 = is_f32(y, "y");
    same_type(y, gate, "gate");
    same_type(y, out, "out");
    const int64_t T = y.size(0), W = y.size(1);
    TORCH_CHECK(y.dim() == 2 && y.is_contiguous() && heads > 0 && W % heads == 0);
    check_rows(out, T, W, "out");
    check_rows(gate, T, W, "gate");
    const int64_t gs = W / heads;
    const bool v = vec8({&out, &y, &gate, &w}, {gs});
    if (v && gs <= 512)
        CHECK_HIP(launch_head_norm(out.data_ptr(), out.stride(0), y.data_ptr(), gate.data_ptr(),
                                   gate.stride(0), f32_ptr(w, W, "w"), (float)eps, heads, gs,
                                   sigmoid, T, f32, current_stream()));
    else
        CHECK_HIP(launch_gated_norm(out.data_ptr(), out.stride(0), y.data_ptr(),
                                    gate.data_ptr(), gate.stride(0), f32_ptr(w, W, "w"),
                                    (float)eps, heads, gs, sigmoid ? 0 : 2, T, f32, v,
                                    current_stream()));
}

void page_write(Tensor k, Tensor v, Tensor k_pages, Tensor v_pages, Tensor slot_mapping) {
    const bool f32 = is_f32(k, "k");
    same_type(k, v, "v");
    same_type(k, k_pages, "k_pages");
    same_type(k, v_pages, "v_pages");
    const int64_t T = k.size(0), wk = k.size(1), wv = v.size(1);
    check_rows(k, T, wk, "k");
    check_rows(v, T, wv, "v");
    TORCH_CHECK(k_pages.dim() == 3 && k_pages.is_contiguous() && k_pages.size(2) == wk);
    TORCH_CHECK(v_pages.dim() == 3 && v_pages.is_contiguous() && v_pages.size(2) == wv);
    CHECK_HIP(launch_page_write(k_pages.data_ptr(), v_pages.data_ptr(), k.data_ptr(),
                                k.stride(0), v.data_ptr(), v.stride(0),
                                i64_ptr(slot_mapping, T, "slots"), T, wk, wv, f32,
                                vec8({&k, &v, &k_pages, &v_pages}, {wk, wv}),
                                current_stream()));
}

struct PagedShapes {
    int64_t T, dim, vdim;
    bool f32, vec;
};
PagedShapes check_paged(const Tensor& out, const Tensor& q, const Tensor& k, const Tensor& v,
                        int64_t H, int64_t G, const Tensor& gate, double cap) {
    PagedShapes s;
    s.f32 = is_f32(q, "q");
    for (const Tensor* t : {&out, &k, &v, &gate}) same_type(q, *t, "attention");
    TORCH_CHECK(G > 0 && H % G == 0 && cap > 0);
    TORCH_CHECK(k.dim() == 3 && k.is_contiguous() && v.dim() == 3 && v.is_contiguous() &&
                k.size(2) % G == 0 && v.size(2) % G == 0 && k.size(0) == v.size(0) &&
                k.size(1) == v.size(1));
    s.T = q.size(0);
    s.dim = k.size(2) / G;
    s.vdim = v.size(2) / G;
    check_rows(q, s.T, H * s.dim, "q");
    check_rows(out, s.T, H * s.vdim, "out");
    check_rows(gate, s.T, H, "gate");
    s.vec = vec8({&q, &k, &v, &out}, {s.dim, s.vdim});
    return s;
}

// nsplit 0: the any-size form; rows: which rows of the batch (all by default)
void paged_rows(Tensor out, Tensor q, Tensor k, Tensor v, int64_t H, int64_t G, Tensor sink,
                double scale, double cap, Tensor gate, double out_scale, Tensor positions,
                Tensor row_seg, Tensor tables, OptTensor rows, int64_t nsplit,
                OptTensor part_acc, OptTensor part_ml) {
    const PagedShapes s = check_paged(out, q, k, v, H, G, gate, cap);
    TORCH_CHECK(tables.dim() == 2);
    const int64_t n = has(rows) ? rows->numel() : s.T;
    float *pa = nullptr, *pm = nullptr;
    if (nsplit > 0) TORCH_CHECK(!s.f32 && s.vec, "paged rows: sizes of the MFMA form");
    if (nsplit > 1) {
        TORCH_CHECK(has(part_acc) && has(part_ml));
        TORCH_CHECK(part_acc->numel() >= n * H * nsplit * s.vdim &&
                    part_ml->numel() >= n * H * nsplit * 2, "paged rows: scratch too small");
        f32_ptr(*part_acc, part_acc->numel(), "part_acc");
        f32_ptr(*part_ml, part_ml->numel(), "part_ml");
        pa = part_acc->data_ptr<float>();
        pm = part_ml->data_ptr<float>();
    }
    CHECK_HIP(launch_paged_rows(
        out.data_ptr(), out.stride(0), q.data_ptr(), q.stride(0), k.data_ptr(), v.data_ptr(),
        f32_ptr(sink, H, "sink"), gate.data_ptr(), gate.stride(0), (float)scale, (float)cap,
        (float)out_scale, i64_ptr(positions, s.T, "positions"), i32_ptr(row_seg, s.T, "row_seg"),
        i32_ptr(tables, 1, "tables"), has(rows) ? i32_ptr(*rows, n, "rows") : nullptr,
        tables.size(1), k.size(1), H, G, s.dim, s.vdim, n, nsplit, pa, pm, s.f32,
        current_stream()));
}

void paged_tiles(Tensor out, Tensor q, Tensor k, Tensor v, int64_t H, int64_t G, Tensor sink,
                 double scale, double cap, Tensor gate, double out_scale, Tensor positions,
                 Tensor tables, Tensor cu, Tensor tile_seg, Tensor tile_off,
                 int64_t tile_rows) {
    const PagedShapes s = check_paged(out, q, k, v, H, G, gate, cap);
    TORCH_CHECK(!s.f32 && s.vec && tables.dim() == 2);
    const int64_t nt = tile_seg.numel();
    CHECK_HIP(launch_paged_tiles(
        out.data_ptr(), out.stride(0), q.data_ptr(), q.stride(0), k.data_ptr(), v.data_ptr(),
        f32_ptr(sink, H, "sink"), gate.data_ptr(), gate.stride(0), (float)scale, (float)cap,
        (float)out_scale, i64_ptr(positions, s.T, "positions"), i32_ptr(tables, 1, "tables"),
        tables.size(1), k.size(1), H, G, s.dim, s.vdim, i32_ptr(cu, 2, "cu"),
        i32_ptr(tile_seg, nt, "tile_seg"), i32_ptr(tile_off, nt, "tile_off"), nt, tile_rows,
        current_stream()));
}

// kind 0: log sigmoid(z) / tau, 1: -e^z, 2: -rate softplus(z)
void decay_logs(Tensor out, Tensor a, Tensor w2, Tensor bias, int64_t kind, double tau,
                OptTensor rate) {
    const bool f32 = is_f32(a, "a");
    same_type(a, w2, "w2");
    TORCH_CHECK(w2.dim() == 2 && w2.is_contiguous() && tau > 0);
    TORCH_CHECK(kind >= 0 && kind <= 2 && has(rate) == (kind == 2));
    const int64_t T = a.size(0), N = w2.size(0), R = w2.size(1);
    check_rows(a, T, R, "a");
    f32_ptr(out, T * N, "out");
    const bool v = vec8({&a, &w2}, {R}) && N % 4 == 0 &&
                   reinterpret_cast<uintptr_t>(bias.data_ptr()) % 16 == 0 &&
                   (kind != 2 || reinterpret_cast<uintptr_t>(rate->data_ptr()) % 16 == 0);
    CHECK_HIP(launch_decay_logs(out.data_ptr<float>(), a.data_ptr(), a.stride(0),
                                w2.data_ptr(), f32_ptr(bias, N, "bias"),
                                kind == 2 ? f32_ptr(*rate, N, "rate") : nullptr, kind,
                                (float)(1.0 / tau), T, N, R, f32, v, current_stream()));
}

struct DecayShapes {
    int64_t T, S;
    bool f32;
    const float* u;
};
DecayShapes check_decay(const Tensor& y, const Tensor& q, const Tensor& k, const Tensor& v,
                        const Tensor& logw, const OptTensor& u, int64_t H, int64_t dk,
                        int64_t dv, const Tensor& state, const Tensor& slots) {
    DecayShapes s;
    s.f32 = is_f32(q, "q");
    for (const Tensor* t : {&y, &k, &v}) same_type(q, *t, "recurrence");
    s.T = q.size(0);
    s.S = slots.numel();
    check_rows(q, s.T, H * dk, "q");
    check_rows(k, s.T, H * dk, "k");
    check_rows(v, s.T, H * dv, "v");
    TORCH_CHECK(y.is_contiguous() && y.numel() == s.T * H * dv);
    f32_ptr(logw, s.T * H * dk, "logw");
    TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == dv &&
                state.size(3) == dk);
    f32_ptr(state, state.numel(), "state");
    TORCH_CHECK(dk <= 512, "recurrence: key size above 512");
    s.u = has(u) ? f32_ptr(*u, H * dk, "u") : nullptr;
    return s;
}

void decay_scan(Tensor y, Tensor q, Tensor k, Tensor v, Tensor logw, OptTensor u, double qscale,
                int64_t H, int64_t dk, int64_t dv, Tensor state, Tensor positions, Tensor cu,
                Tensor slots, OptTensor seg_list) {
    const DecayShapes s = check_decay(y, q, k, v, logw, u, H, dk, dv, state, slots);
    int64_t nseg = s.S;
    const int* list = nullptr;
    if (has(seg_list)) {
        nseg = seg_list->numel();
        list = i32_ptr(*seg_list, 0, "seg_list");
    }
    CHECK_HIP(launch_decay_scan(
        y.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), logw.data_ptr<float>(), s.u, (float)qscale, s.T, H, dk, dv,
        state.data_ptr<float>(), i64_ptr(positions, s.T, "positions"), i32_ptr(cu, s.S + 1, "cu"),
        i32_ptr(slots, s.S, "slots"), list, nseg, s.f32, current_stream()));
}

// logw is overwritten; segs/first/chunk_seg/chunk_off as in the other chunked forms
void decay_chunked(Tensor y, Tensor q, Tensor k, Tensor v, Tensor logw, OptTensor u,
                   double qscale, int64_t H, int64_t dk, int64_t dv, Tensor state,
                   Tensor positions, Tensor cu, Tensor slots, Tensor segs, Tensor first,
                   Tensor chunk_seg, Tensor chunk_off) {
    const DecayShapes s = check_decay(y, q, k, v, logw, u, H, dk, dv, state, slots);
    TORCH_CHECK(!s.f32 && vec8({&q, &k, &v, &y}, {dk, dv}) && dk <= 256);
    if (has(u)) TORCH_CHECK(vec8({&*u}, {}));
    const int64_t L = segs.numel(), nc = chunk_seg.numel();
    auto planes = torch::empty({2, nc, H, dv, dk}, q.options());
    CHECK_HIP(launch_decay_chunked(
        y.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), logw.data_ptr<float>(), s.u, (float)qscale, s.T, H, dk, dv,
        state.data_ptr<float>(), i64_ptr(positions, s.T, "positions"), i32_ptr(cu, s.S + 1, "cu"),
        i32_ptr(slots, s.S, "slots"), i32_ptr(segs, L, "segs"), i32_ptr(first, L + 1, "first"),
        i32_ptr(chunk_seg, nc, "chunk_seg"), i32_ptr(chunk_off, nc, "chunk_off"), L, nc,
        planes.data_ptr(), current_stream()));
}

void clamped_glu(Tensor out, Tensor x, double limit) {
    const bool f32 = is_f32(x, "x");
    same_type(x, out, "out");
    TORCH_CHECK(x.dim() == 2 && x.is_contiguous() && out.is_contiguous());
    const int64_t T = x.size(0), ff = x.size(1) / 2;
    TORCH_CHECK(x.size(1) == 2 * ff && out.numel() == T * ff);
    CHECK_HIP(launch_clamped_glu(out.data_ptr(), x.data_ptr(), (float)limit, T, ff, f32,
                                 vec8({&x, &out}, {ff}), current_stream()));
}

void soft_cap(Tensor x, double cap) {
    TORCH_CHECK(cap > 0);
    f32_ptr(x, x.numel(), "x");
    CHECK_HIP(launch_soft_cap(x.data_ptr<float>(), (float)cap, x.numel(), current_stream()));
}

// z [T, E] logits -> ids, weights [T, top], and the rows' places by expert
void route(Tensor ids, Tensor weights, Tensor slot, Tensor row_token, Tensor tile_info,
           Tensor z, OptTensor bias, double scale, int64_t tile_rows) {
    TORCH_CHECK(z.dim() == 2 && ids.dim() == 2);
    const int64_t T = z.size(0), E = z.size(1), top = ids.size(1), nt = (tile_info.numel() - 1) / 4;
    f32_ptr(z, T * E, "z");
    i32_ptr(ids, T * top, "ids");
    f32_ptr(weights, T * top, "weights");
    i32_ptr(slot, T * top, "slot");
    i32_ptr(tile_info, 4 * nt + 1, "tile_info");
    i32_ptr(row_token, nt * tile_rows, "row_token");
    TORCH_CHECK(reinterpret_cast<uintptr_t>(tile_info.data_ptr()) % 16 == 0, "tile_info: unaligned");
    TORCH_CHECK(tile_rows > 0 && nt >= std::min(T * top, E + T * top / tile_rows),
                "route: too few tiles");
    CHECK_HIP(launch_route_topk(ids.data_ptr<int>(), weights.data_ptr<float>(),
                                z.data_ptr<float>(),
                                has(bias) ? f32_ptr(*bias, E, "bias") : nullptr, (float)scale, T,
                                E, top, current_stream()));
    CHECK_HIP(launch_route_plan(slot.data_ptr<int>(), row_token.data_ptr<int>(),
                                tile_info.data_ptr<int>(), ids.data_ptr<int>(), T * top, top,
                                E, tile_rows, nt, current_stream()));
}

// out[r] = w[e] x[token(r)] through a GLU (glu 1: clamped, 2: silu), or w[e] x[r]
void expert_product(Tensor out, Tensor x, Tensor w, Tensor row_token, Tensor tile_info,
                    int64_t tile_rows, int64_t glu, double limit) {
    const bool f32 = is_f32(x, "x"), frag = w.dim() == 5;
    same_type(x, w, "w");
    same_type(x, out, "out");
    const int64_t nt = (tile_info.numel() - 1) / 4, R = nt * tile_rows;
    const int64_t N = out.size(1), K = x.size(1);
    check_rows(out, R, N, "out");
    check_rows(x, x.size(0), K, "x");
    TORCH_CHECK(reinterpret_cast<uintptr_t>(tile_info.data_ptr()) % 16 == 0, "tile_info: unaligned");
    TORCH_CHECK(glu >= 0 && glu <= 2);
    TORCH_CHECK(x.size(0) > 0 && (glu || x.size(0) == R) && w.is_contiguous());
    int64_t nfrags = 0, ksteps = 0;
    if (frag) {
        TORCH_CHECK(w.size(3) == 64 && w.size(4) == 8 && vec8({&x, &out, &w}, {N, K}));
        nfrags = w.size(1);
        ksteps = w.size(2);
    } else {
        TORCH_CHECK(w.dim() == 3 && w.size(1) == (glu ? 2 : 1) * N && w.size(2) == K);
    }
    CHECK_HIP(launch_expert_product(
        out.data_ptr(), out.stride(0), x.data_ptr(), x.stride(0), w.data_ptr(),
        i32_ptr(row_token, R, "row_token"), i32_ptr(tile_info, 4 * nt + 1, "tile_info"), N, K, glu,
        (float)limit, frag, nfrags, ksteps, tile_rows, nt, f32, current_stream()));
}

}  // namespace

void bind_parallel(pybind11::module_& m) {
    m.def("stream_tanh", &stream_tanh, "stream add + dynamic tanh");
    m.def("embed_tanh", &embed_tanh, "embedding + dynamic tanh into the fp32 stream");
    m.def("token_shift", &token_shift, "mixes of every row with the previous one");
    m.def("head_norm_gate", &head_norm_gate, "head-wise RMS norm with a silu or sigmoid gate");
    m.def("page_write", &page_write, "keys and values into cache pages");
    m.def("paged_rows", &paged_rows, "attention over pages, row by row");
    m.def("paged_tiles", &paged_tiles, "attention over pages, tiles of prompt rows");
    m.def("decay_logs", &decay_logs, "log decays from a low-rank product");
    m.def("decay_scan", &decay_scan, "per-channel-decay recurrence, token by token");
    m.def("decay_chunked", &decay_chunked, "per-channel-decay recurrence, chunked");
    m.def("clamped_glu", &clamped_glu, "clamped GLU");
    m.def("soft_cap", &soft_cap, "cap * tanh(x / cap) in place");
    m.def("route", &route, "top-k routing, rows grouped by expert");
    m.def("expert_product", &expert_product, "one product of the grouped experts");
}
