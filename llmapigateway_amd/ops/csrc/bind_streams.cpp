// Bindings of the hyper-connected streams, rotary attention in a window, fixed
// decays and the delta rule (the rest of the hybrid kernels: ext_hybrid.cpp).
// Shapes, strides and dtypes are checked here.

#include "bind_shared.h"
#include "bind_checks.h"

extern "C" {
hipError_t launch_mix_streams(void*, float*, const float*, const void* const*, const float* const*, const float*, const float*, float, int, int, int, int, int, int, int, hipStream_t);
hipError_t launch_embed_rms(float*, const int64_t*, const void*, const float*, float, int, int, int, int, hipStream_t);
hipError_t launch_xielu(void*, float, float, size_t, int, int, hipStream_t);
hipError_t launch_silu(void*, int64_t, int, int, int, int, hipStream_t);
hipError_t launch_rotary_rows(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, const float*, const float*, float, const float*, const int64_t*, void*, void*, const int64_t*, int, int, int, int, int, int, int, int, hipStream_t);
hipError_t launch_window_rows(void*, int64_t, const void*, int64_t, const void*, const void*, int, float, int, int, float, float, float, const int64_t*, const int*, const int*, const int*, int, int, int, int, int, int, int, int, float*, float*, int, hipStream_t);
hipError_t launch_window_tiles(void*, int64_t, const void*, int64_t, const void*, const void*, int, float, int, int, float, float, float, const int64_t*, const int*, int, int, int, int, int, int, const int*, const int*, const int*, int, int, hipStream_t);
hipError_t launch_fixed_scan(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, const float*, int, int, int, float*, const int64_t*, const int*, const int*, const int*, int, int, hipStream_t);
hipError_t launch_fixed_chunked(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, const float*, int, int, int, int, float*, const int64_t*, const int*, const int*, const int*, const int*, const int*, const int*, int, int, float*, void*, hipStream_t);
hipError_t launch_delta_scan(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, float*, const void*, int64_t, int, int, int, int, int, float*, const int64_t*, const int*, const int*, const int*, int, int, hipStream_t);
hipError_t launch_delta_chunked(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, float*, const void*, int64_t, int, int, int, int, int, float*, const int64_t*, const int*, const int*, const int*, const int*, const int*, const int*, int, int, void*, float*, hipStream_t);
hipError_t launch_decay_sums(float*, int, const int*, const int*, const int*, int, hipStream_t);
int delta_slices(int);
}

namespace {

// rows x[:, s] and the outputs y (times their scales), combined by coef; h =
// RMS norm of column 0 times w, out = the other columns (may be x)
void mix_streams(Tensor h, OptTensor out, Tensor x, std::vector<Tensor> y,
                 std::vector<OptTensor> scales, Tensor coef, Tensor w, double eps) {
    const bool f32 = is_f32(h, "h");
    TORCH_CHECK(x.dim() == 3 && h.dim() == 2 && h.is_contiguous());
    const int64_t T = x.size(0), S = x.size(1), W = x.size(2), n = y.size();
    f32_ptr(x, T * S * W, "x");
    check_rows(h, T, W, "h");
    TORCH_CHECK(n <= 8 && scales.size() == y.size(), "mix_streams: at most 8 pending outputs");
    TORCH_CHECK(coef.dim() == 2 && coef.size(0) == S + n, "coef: a row for each input");
    const int64_t C = coef.size(1);
    TORCH_CHECK(C >= 1 && C <= 17 && (C > 1) == has(out), "coef: columns");
    bool v = vec8({&h, &x, &w}, {W});
    if (has(out)) {
        f32_ptr(*out, T * (C - 1) * W, "out");
        v = v && vec8({&*out}, {});
        TORCH_CHECK(out->data_ptr() != x.data_ptr() || C - 1 == S, "mix_streams: not in place");
    }
    const void* yp[8] = {};
    const float* sp[8] = {};
    for (int64_t i = 0; i < n; ++i) {
        same_type(y[i], h, "y");
        check_rows(y[i], T, W, "y");
        TORCH_CHECK(y[i].is_contiguous());
        v = v && vec8({&y[i]}, {});
        yp[i] = y[i].data_ptr();
        if (has(scales[i])) {
            sp[i] = f32_ptr(*scales[i], W, "scale");
            v = v && vec8({&*scales[i]}, {});
        }
    }
    CHECK_HIP(launch_mix_streams(
        h.data_ptr(), has(out) ? out->data_ptr<float>() : nullptr, x.data_ptr<float>(), yp, sp,
        f32_ptr(coef, (S + n) * C, "coef"), f32_ptr(w, W, "w"), (float)eps, T, S, n, C, W, f32, v,
        current_stream()));
}

void embed_rms_norm(Tensor x, Tensor tokens, Tensor embed, Tensor w, double eps) {
    const bool f32 = is_f32(embed, "embed");
    TORCH_CHECK(embed.dim() == 2 && embed.is_contiguous());
    const int64_t W = embed.size(1), T = tokens.numel();
    f32_ptr(x, T * W, "x");
    CHECK_HIP(launch_embed_rms(x.data_ptr<float>(), i64_ptr(tokens, T, "tokens"),
                               embed.data_ptr(), f32_ptr(w, W, "w"), (float)eps, T, W, f32,
                               vec8({&x, &embed, &w}, {W}), current_stream()));
}

void xielu(Tensor z, double pos, double neg) {
    const bool f32 = is_f32(z, "z");
    TORCH_CHECK(z.is_contiguous());
    CHECK_HIP(launch_xielu(z.data_ptr(), (float)pos, (float)neg, z.numel(), f32,
                           vec8({&z}, {z.numel()}), current_stream()));
}

void silu(Tensor x) {
    const bool f32 = is_f32(x, "x");
    TORCH_CHECK(x.dim() == 2);
    check_rows(x, x.size(0), x.size(1), "x");
    CHECK_HIP(launch_silu(x.data_ptr(), x.stride(0), x.size(0), x.size(1), f32,
                          vec8({&x}, {x.size(1)}), current_stream()));
}

// heads of q (to out) and k (to the pages): norm and rotation in halves; values
// to the pages
void rotary_rows(Tensor out, Tensor q, OptTensor k, OptTensor v, Tensor q_norm,
                 OptTensor k_norm, double eps, Tensor cos_sin, Tensor positions,
                 OptTensor k_pages, OptTensor v_pages, OptTensor slot_mapping) {
    const bool f32 = is_f32(q, "q");
    same_type(q, out, "out");
    const int64_t T = q.size(0), dim = q_norm.numel(), wq = q.size(1);
    TORCH_CHECK(dim > 0 && wq % dim == 0);
    check_rows(q, T, wq, "q");
    check_rows(out, T, wq, "out");
    TORCH_CHECK(out.is_contiguous());
    TORCH_CHECK(cos_sin.dim() == 2 && cos_sin.size(1) % 2 == 0 && cos_sin.size(1) <= dim);
    const int64_t half = cos_sin.size(1) / 2;
    bool vec = vec8({&q, &out, &q_norm, &cos_sin}, {dim, half});
    int64_t wk = 0, wv = 0;
    if (has(k)) {
        TORCH_CHECK(has(v) && has(k_norm) && has(k_pages) && has(v_pages) && has(slot_mapping));
        wk = k->size(1);
        wv = v->size(1);
        for (const Tensor* t : {&*k, &*v, &*k_pages, &*v_pages}) same_type(q, *t, "rotary_rows");
        check_rows(*k, T, wk, "k");
        check_rows(*v, T, wv, "v");
        TORCH_CHECK(wk % dim == 0 && k_norm->numel() == dim);
        TORCH_CHECK(k_pages->dim() == 3 && k_pages->is_contiguous() && k_pages->size(2) == wk);
        TORCH_CHECK(v_pages->dim() == 3 && v_pages->is_contiguous() && v_pages->size(2) == wv);
        vec = vec && vec8({&*k, &*v, &*k_norm, &*k_pages, &*v_pages}, {wv});
    }
    CHECK_HIP(launch_rotary_rows(
        out.data_ptr(), q.data_ptr(), q.stride(0), has(k) ? k->data_ptr() : nullptr,
        has(k) ? k->stride(0) : 0, has(k) ? v->data_ptr() : nullptr, has(k) ? v->stride(0) : 0,
        f32_ptr(q_norm, dim, "q_norm"), has(k) ? f32_ptr(*k_norm, dim, "k_norm") : nullptr,
        (float)eps, f32_ptr(cos_sin, cos_sin.numel(), "cos_sin"),
        i64_ptr(positions, T, "positions"), has(k) ? k_pages->data_ptr() : nullptr,
        has(k) ? v_pages->data_ptr() : nullptr,
        has(k) ? i64_ptr(*slot_mapping, T, "slots") : nullptr, T, wq / dim, wk / dim, dim, half,
        wv, f32, vec, current_stream()));
}

struct WindowShapes {
    int64_t T, dim, vdim;
    bool f32, vec;
};
WindowShapes check_window(const Tensor& out, const Tensor& q, const Tensor& k, const Tensor& v,
                          int64_t H, int64_t G, int64_t maps, int64_t window, int64_t keep) {
    WindowShapes s;
    s.f32 = is_f32(q, "q");
    for (const Tensor* t : {&out, &k, &v}) same_type(q, *t, "attention");
    TORCH_CHECK(G > 0 && H % G == 0 && (maps == 1 || maps == 2));
    TORCH_CHECK(window >= 1 && window <= 1 << 30 && keep >= 0 && keep <= 1 << 30);
    TORCH_CHECK(k.dim() == 3 && k.is_contiguous() && v.dim() == 3 && v.is_contiguous() &&
                k.size(2) % (G * maps) == 0 && v.size(2) % G == 0 && k.size(0) == v.size(0) &&
                k.size(1) == v.size(1));
    s.T = q.size(0);
    s.dim = k.size(2) / (G * maps);
    s.vdim = v.size(2) / G;
    check_rows(q, s.T, H * maps * s.dim, "q");
    check_rows(out, s.T, H * s.vdim, "out");
    s.vec = vec8({&q, &k, &v, &out}, {s.dim, s.vdim});
    return s;
}

// nsplit 0: the any-size form; rows: which rows of the batch (all by default)
void window_rows(Tensor out, Tensor q, Tensor k, Tensor v, int64_t H, int64_t G, int64_t maps,
                 double scale, int64_t window, int64_t keep, double lam, double gain, double eps,
                 Tensor positions, Tensor row_seg, Tensor tables, OptTensor rows, int64_t nsplit,
                 OptTensor part_acc, OptTensor part_ml) {
    const WindowShapes s = check_window(out, q, k, v, H, G, maps, window, keep);
    TORCH_CHECK(tables.dim() == 2);
    const int64_t n = has(rows) ? rows->numel() : s.T;
    float *pa = nullptr, *pm = nullptr;
    if (nsplit > 0) TORCH_CHECK(!s.f32 && s.vec, "window rows: sizes of the MFMA form");
    if (nsplit > 1) {
        TORCH_CHECK(has(part_acc) && has(part_ml));
        TORCH_CHECK(part_acc->numel() >= n * H * maps * nsplit * s.vdim &&
                    part_ml->numel() >= n * H * maps * nsplit * 2, "window rows: scratch too small");
        f32_ptr(*part_acc, part_acc->numel(), "part_acc");
        f32_ptr(*part_ml, part_ml->numel(), "part_ml");
        pa = part_acc->data_ptr<float>();
        pm = part_ml->data_ptr<float>();
    }
    CHECK_HIP(launch_window_rows(
        out.data_ptr(), out.stride(0), q.data_ptr(), q.stride(0), k.data_ptr(), v.data_ptr(),
        maps, (float)scale, window, keep, (float)lam, (float)gain, (float)eps,
        i64_ptr(positions, s.T, "positions"), i32_ptr(row_seg, s.T, "row_seg"),
        i32_ptr(tables, 1, "tables"), has(rows) ? i32_ptr(*rows, n, "rows") : nullptr,
        tables.size(1), k.size(1), H, G, s.dim, s.vdim, n, nsplit, pa, pm, s.f32,
        current_stream()));
}

void window_tiles(Tensor out, Tensor q, Tensor k, Tensor v, int64_t H, int64_t G, int64_t maps,
                  double scale, int64_t window, int64_t keep, double lam, double gain,
                  double eps, Tensor positions, Tensor tables, Tensor cu, Tensor tile_seg,
                  Tensor tile_off, int64_t tile_rows) {
    const WindowShapes s = check_window(out, q, k, v, H, G, maps, window, keep);
    TORCH_CHECK(!s.f32 && s.vec && tables.dim() == 2);
    const int64_t nt = tile_seg.numel();
    CHECK_HIP(launch_window_tiles(
        out.data_ptr(), out.stride(0), q.data_ptr(), q.stride(0), k.data_ptr(), v.data_ptr(),
        maps, (float)scale, window, keep, (float)lam, (float)gain, (float)eps,
        i64_ptr(positions, s.T, "positions"), i32_ptr(tables, 1, "tables"), tables.size(1),
        k.size(1), H, G, s.dim, s.vdim, i32_ptr(cu, 2, "cu"), i32_ptr(tile_seg, nt, "tile_seg"),
        i32_ptr(tile_off, nt, "tile_off"), nt, tile_rows, current_stream()));
}

struct StateShapes {
    int64_t T, S;
    bool f32;
};
StateShapes check_state(const Tensor& y, const Tensor& q, const Tensor& k, const Tensor& v,
                        int64_t H, int64_t G, int64_t dk, int64_t dv, const Tensor& state,
                        const Tensor& slots) {
    StateShapes s;
    s.f32 = is_f32(q, "q");
    for (const Tensor* t : {&y, &k, &v}) same_type(q, *t, "recurrence");
    s.T = q.size(0);
    s.S = slots.numel();
    TORCH_CHECK(G > 0 && H % G == 0);
    check_rows(q, s.T, G * dk, "q");
    check_rows(k, s.T, G * dk, "k");
    check_rows(v, s.T, H * dv, "v");
    TORCH_CHECK(y.is_contiguous() && y.numel() == s.T * H * dv);
    TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == dv &&
                state.size(3) == dk);
    f32_ptr(state, state.numel(), "state");
    TORCH_CHECK(dk <= 512, "recurrence: key size above 512");
    return s;
}
const int* listed(const OptTensor& list, int64_t all, int64_t& n) {
    n = has(list) ? list->numel() : all;
    return has(list) ? i32_ptr(*list, 0, "seg_list") : nullptr;
}

void fixed_scan(Tensor y, Tensor q, Tensor k, Tensor v, Tensor decay, int64_t H, int64_t dk,
                int64_t dv, Tensor state, Tensor positions, Tensor cu, Tensor slots,
                OptTensor seg_list) {
    const StateShapes s = check_state(y, q, k, v, H, H, dk, dv, state, slots);
    int64_t nseg;
    const int* list = listed(seg_list, s.S, nseg);
    CHECK_HIP(launch_fixed_scan(
        y.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), f32_ptr(decay, H, "decay"), H, dk, dv, state.data_ptr<float>(),
        i64_ptr(positions, s.T, "positions"), i32_ptr(cu, s.S + 1, "cu"),
        i32_ptr(slots, s.S, "slots"), list, nseg, s.f32, current_stream()));
}

// q, k and v went through silu; segs/first/chunk_seg/chunk_off as in the other
// chunked forms
void fixed_chunked(Tensor y, Tensor q, Tensor k, Tensor v, Tensor decay, int64_t H, int64_t dk,
                   int64_t dv, Tensor state, Tensor positions, Tensor cu, Tensor slots,
                   Tensor segs, Tensor first, Tensor chunk_seg, Tensor chunk_off) {
    const StateShapes s = check_state(y, q, k, v, H, H, dk, dv, state, slots);
    TORCH_CHECK(!s.f32 && vec8({&q, &k, &v, &y}, {dk, dv}));
    const int64_t L = segs.numel(), nc = chunk_seg.numel();
    auto Fb = torch::empty({2, H, s.T}, q.options().dtype(torch::kFloat32));
    auto planes = torch::empty({2, nc, H, dv, dk}, q.options());
    CHECK_HIP(launch_fixed_chunked(
        y.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), f32_ptr(decay, H, "decay"), s.T, H, dk, dv, state.data_ptr<float>(),
        i64_ptr(positions, s.T, "positions"), i32_ptr(cu, s.S + 1, "cu"),
        i32_ptr(slots, s.S, "slots"), i32_ptr(segs, L, "segs"), i32_ptr(first, L + 1, "first"),
        i32_ptr(chunk_seg, nc, "chunk_seg"), i32_ptr(chunk_off, nc, "chunk_off"), L, nc,
        Fb.data_ptr<float>(), planes.data_ptr(), current_stream()));
}

void delta_scan(Tensor y, Tensor q, Tensor k, Tensor v, Tensor logw, Tensor b, int64_t H,
                int64_t G, int64_t dk, int64_t dv, Tensor state, Tensor positions, Tensor cu,
                Tensor slots, OptTensor seg_list) {
    const StateShapes s = check_state(y, q, k, v, H, G, dk, dv, state, slots);
    same_type(q, b, "b");
    check_rows(b, s.T, H, "b");
    f32_ptr(logw, s.T * H * dk, "logw");
    int64_t nseg;
    const int* list = listed(seg_list, s.S, nseg);
    CHECK_HIP(launch_delta_scan(
        y.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), logw.data_ptr<float>(), b.data_ptr(), b.stride(0), s.T, H, G, dk, dv,
        state.data_ptr<float>(), i64_ptr(positions, s.T, "positions"), i32_ptr(cu, s.S + 1, "cu"),
        i32_ptr(slots, s.S, "slots"), list, nseg, s.f32, current_stream()));
}

// logw is overwritten
void delta_chunked(Tensor y, Tensor q, Tensor k, Tensor v, Tensor logw, Tensor b, int64_t H,
                   int64_t G, int64_t dk, int64_t dv, Tensor state, Tensor positions, Tensor cu,
                   Tensor slots, Tensor segs, Tensor first, Tensor chunk_seg,
                   Tensor chunk_off) {
    const StateShapes s = check_state(y, q, k, v, H, G, dk, dv, state, slots);
    same_type(q, b, "b");
    check_rows(b, s.T, H, "b");
    f32_ptr(logw, s.T * H * dk, "logw");
    TORCH_CHECK(!s.f32 && vec8({&q, &k, &v, &y, &logw}, {dk, dv}) && dk <= 256);
    const int64_t L = segs.numel(), nc = chunk_seg.numel(), NC = delta_slices(dk);
    auto frags = torch::empty({nc, H, 3 * NC + 2, 4096}, q.options());
    auto u0 = torch::empty({nc, H, (dv + 31) / 32, 2048}, logw.options());
    const int* cp = i32_ptr(cu, s.S + 1, "cu");
    const int *seg = i32_ptr(chunk_seg, nc, "chunk_seg"), *off = i32_ptr(chunk_off, nc, "chunk_off");
    CHECK_HIP(launch_decay_sums(logw.data_ptr<float>(), H * dk, cp, seg, off, nc, current_stream()));
    CHECK_HIP(launch_delta_chunked(
        y.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), logw.data_ptr<float>(), b.data_ptr(), b.stride(0), s.T, H, G, dk, dv,
        state.data_ptr<float>(), i64_ptr(positions, s.T, "positions"), cp,
        i32_ptr(slots, s.S, "slots"), i32_ptr(segs, L, "segs"), i32_ptr(first, L + 1, "first"),
        seg, off, L, nc, frags.data_ptr(), u0.data_ptr<float>(), current_stream()));
}

}  // namespace

void bind_streams(pybind11::module_& m) {
    m.def("mix_streams", &mix_streams, "streams and pending outputs combined, with a norm");
    m.def("embed_rms_norm", &embed_rms_norm, "embedding + RMS norm into the fp32 stream");
    m.def("xielu", &xielu, "xIELU in place");
    m.def("silu", &silu, "silu in place");
    m.def("rotary_rows", &rotary_rows, "head norms + rotation in halves + page write");
    m.def("window_rows", &window_rows, "softmax attention in a window, row by row");
    m.def("window_tiles", &window_tiles, "softmax attention in a window, tiles of prompt rows");
    m.def("fixed_scan", &fixed_scan, "fixed-decay recurrence, token by token");
    m.def("fixed_chunked", &fixed_chunked, "fixed-decay recurrence, chunked");
    m.def("delta_scan", &delta_scan, "channel-decay delta rule, token by token");
    m.def("delta_chunked", &delta_chunked, "channel-decay delta rule, chunked");
}
