// Bindings of the RMS-norm rows and of sigmoid attention over pages with mixed
// heads (the rest of the hybrid kernels: ext_hybrid.cpp). Shapes, strides and
// dtypes are checked here.

#include "bind_shared.h"
#include "bind_checks.h"

extern "C" {
hipError_t launch_add_rms_norm(void*, void*, float*, const void*, const void*, const void*, const int*, const float*, int, const float*, const float*, float, int, int, int, int, hipStream_t);
hipError_t launch_qkv_rows(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, const void*, int64_t, const float*, const float*, float, float, void*, void*, const int64_t*, int, int, int, int, int, int, hipStream_t);
hipError_t launch_sigmoid_rows(void*, int64_t, const void*, int64_t, const void*, const void*, const float*, const void*, const void*, int64_t, float, const int64_t*, const int*, const int*, const int*, int, int, int, int, int, int, int, int, int, int, int, float*, int, hipStream_t);
hipError_t launch_sigmoid_tiles(void*, int64_t, const void*, int64_t, const void*, const void*, const float*, const void*, const void*, int64_t, float, const int64_t*, const int*, int, int, int, int, int, int, int, int, int, const int*, const int*, const int*, int, hipStream_t);
}

namespace {

// x (fp32 stream) += d1 + d2 + the experts' sum (each optional); out1 and
// out2 = RMS norm(x) times w1 and w2
void add_rms_norm(Tensor out1, OptTensor out2, Tensor x, OptTensor d1, OptTensor d2,
                  OptTensor rows, OptTensor slot, OptTensor weights, Tensor w1, OptTensor w2,
                  double eps) {
    const bool f32 = is_f32(out1, "out1");
    TORCH_CHECK(x.dim() == 2);
    const int64_t T = x.size(0), W = x.size(1);
    f32_ptr(x, T * W, "x");
    bool v = vec8({&x, &w1}, {W});
    auto dense = [&](const OptTensor& t, const char* name) -> void* {
        if (!has(t)) return nullptr;
        same_type(*t, out1, name);
        check_rows(*t, T, W, name);
        TORCH_CHECK(t->is_contiguous(), name, ": dense");
        v = v && vec8({&*t}, {});
        return t->data_ptr();
    };
    void *o1 = dense(out1, "out1"), *o2 = dense(out2, "out2");
    const void *p1 = dense(d1, "d1"), *p2 = dense(d2, "d2"), *rp = nullptr;
    TORCH_CHECK(p1 || !p2, "add_rms_norm: d2 without d1");
    TORCH_CHECK(has(out2) == has(w2));
    const int* ip = nullptr;
    const float* wp = nullptr;
    int64_t top = 0;
    if (has(slot)) {
        TORCH_CHECK(has(rows) && has(weights) && slot->dim() == 2);
        same_type(*rows, out1, "rows");
        check_rows(*rows, rows->size(0), W, "rows");
        TORCH_CHECK(rows->is_contiguous());
        top = slot->size(1);
        ip = i32_ptr(*slot, T * top, "slot");
        wp = f32_ptr(*weights, T * top, "weights");
        rp = rows->data_ptr();
        v = v && vec8({&*rows}, {});
    }
    if (has(w2)) v = v && vec8({&*w2}, {});
    CHECK_HIP(launch_add_rms_norm(o1, o2, x.data_ptr<float>(), p1, p2, rp, ip, wp, top,
                                  f32_ptr(w1, W, "w1"), has(w2) ? f32_ptr(*w2, W, "w2") : nullptr,
                                  (float)eps, T, W, f32, v, current_stream()));
}

// out = RMS norm of whole rows of q; keys (normed alike) and values (blended
// with v_first) into their cache slots
void qkv_rows(Tensor out, Tensor q, Tensor k, Tensor v, Tensor q_norm, Tensor k_norm, double eps,
              double blend, OptTensor v_first, Tensor k_pages, Tensor v_pages,
              Tensor slot_mapping) {
    const bool f32 = is_f32(q, "q");
    for (const Tensor* t : {&out, &k, &v, &k_pages, &v_pages}) same_type(q, *t, "qkv_rows");
    const int64_t T = q.size(0), wq = q.size(1), wk = k.size(1), wv = v.size(1);
    check_rows(q, T, wq, "q");
    check_rows(k, T, wk, "k");
    check_rows(v, T, wv, "v");
    check_rows(out, T, wq, "out");
    TORCH_CHECK(out.is_contiguous());
    TORCH_CHECK(k_pages.dim() == 3 && k_pages.is_contiguous() && k_pages.size(2) == wk);
    TORCH_CHECK(v_pages.dim() == 3 && v_pages.is_contiguous() && v_pages.size(2) == wv);
    bool vec = vec8({&q, &k, &v, &out, &q_norm, &k_norm, &k_pages, &v_pages}, {wq, wk, wv});
    if (has(v_first)) {
        same_type(q, *v_first, "v_first");
        check_rows(*v_first, T, wv, "v_first");
        vec = vec && vec8({&*v_first}, {});
    }
    CHECK_HIP(launch_qkv_rows(
        out.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), has(v_first) ? v_first->data_ptr() : nullptr,
        has(v_first) ? v_first->stride(0) : 0, f32_ptr(q_norm, wq, "q_norm"),
        f32_ptr(k_norm, wk, "k_norm"), (float)eps, (float)blend, k_pages.data_ptr(),
        v_pages.data_ptr(), i64_ptr(slot_mapping, T, "slots"), T, wq, wk, wv, f32, vec,
        current_stream()));
}

struct SigmoidShapes {
    int64_t T, dim, vdim, nbias, Hp;
    bool f32, vec;
    const float* bias;
};
SigmoidShapes check_sigmoid(const Tensor& out, const Tensor& q, const Tensor& k, const Tensor& v,
                            int64_t H, int64_t G, const Tensor& bias, const Tensor& talk,
                            int64_t window, const Tensor& gate) {
    SigmoidShapes s;
    s.f32 = is_f32(q, "q");
    for (const Tensor* t : {&out, &k, &v, &gate, &talk}) same_type(q, *t, "attention");
    TORCH_CHECK(G > 0 && H % G == 0 && window > 0);
    TORCH_CHECK(k.dim() == 3 && k.is_contiguous() && v.dim() == 3 && v.is_contiguous() &&
                k.size(2) % G == 0 && v.size(2) % G == 0 && k.size(0) == v.size(0) &&
                k.size(1) == v.size(1));
    TORCH_CHECK(talk.is_contiguous() && talk.numel() == H * H, "talk: [H, H]");
    TORCH_CHECK(bias.dim() == 2 && bias.size(0) > 0 && bias.size(1) >= H, "bias: [distances, H]");
    s.nbias = bias.size(0);
    s.Hp = bias.size(1);
    s.bias = f32_ptr(bias, s.nbias * s.Hp, "bias");
    s.T = q.size(0);
    s.dim = k.size(2) / G;
    s.vdim = v.size(2) / G;
    check_rows(q, s.T, H * s.dim, "q");
    check_rows(out, s.T, H * s.vdim, "out");
    check_rows(gate, s.T, H * s.vdim, "gate");
    s.vec = vec8({&q, &k, &v, &out, &gate, &bias}, {s.dim, s.vdim});
    return s;
}

// nsplit 0: the any-size form; rows: which rows of the batch (all by default)
void sigmoid_rows(Tensor out, Tensor q, Tensor k, Tensor v, int64_t H, int64_t G, double scale,
                  Tensor bias, Tensor talk, int64_t window, Tensor gate, Tensor positions,
                  Tensor row_seg, Tensor tables, OptTensor rows, int64_t nsplit,
                  OptTensor part) {
    const SigmoidShapes s = check_sigmoid(out, q, k, v, H, G, bias, talk, window, gate);
    TORCH_CHECK(tables.dim() == 2);
    const int64_t n = has(rows) ? rows->numel() : s.T;
    float* pp = nullptr;
    if (nsplit > 0) TORCH_CHECK(!s.f32 && s.vec, "sigmoid rows: sizes of the MFMA form");
    if (nsplit > 1) {
        TORCH_CHECK(has(part) && part->numel() >= n * H * nsplit * s.vdim,
                    "sigmoid rows: scratch too small");
        f32_ptr(*part, part->numel(), "part");
        pp = part->data_ptr<float>();
    }
    CHECK_HIP(launch_sigmoid_rows(
        out.data_ptr(), out.stride(0), q.data_ptr(), q.stride(0), k.data_ptr(), v.data_ptr(),
        s.bias, talk.data_ptr(), gate.data_ptr(), gate.stride(0), (float)scale,
        i64_ptr(positions, s.T, "positions"), i32_ptr(row_seg, s.T, "row_seg"),
        i32_ptr(tables, 1, "tables"), has(rows) ? i32_ptr(*rows, n, "rows") : nullptr, window,
        s.nbias, s.Hp, tables.size(1), k.size(1), H, G, s.dim, s.vdim, n, nsplit, pp, s.f32,
        current_stream()));
}

void sigmoid_tiles(Tensor out, Tensor q, Tensor k, Tensor v, int64_t H, int64_t G, double scale,
                   Tensor bias, Tensor talk, int64_t window, Tensor gate, Tensor positions,
                   Tensor tables, Tensor cu, Tensor tile_seg, Tensor tile_off) {
    const SigmoidShapes s = check_sigmoid(out, q, k, v, H, G, bias, talk, window, gate);
    TORCH_CHECK(!s.f32 && s.vec && tables.dim() == 2);
    const int64_t nt = tile_seg.numel();
    CHECK_HIP(launch_sigmoid_tiles(
        out.data_ptr(), out.stride(0), q.data_ptr(), q.stride(0), k.data_ptr(), v.data_ptr(),
        s.bias, talk.data_ptr(), gate.data_ptr(), gate.stride(0), (float)scale,
        i64_ptr(positions, s.T, "positions"), i32_ptr(tables, 1, "tables"), window, s.nbias,
        s.Hp, tables.size(1), k.size(1), H, G, s.dim, s.vdim, i32_ptr(cu, 2, "cu"),
        i32_ptr(tile_seg, nt, "tile_seg"), i32_ptr(tile_off, nt, "tile_off"), nt,
        current_stream()));
}

}  // namespace

void bind_sigmoid(pybind11::module_& m) {
    m.def("add_rms_norm", &add_rms_norm, "stream adds + one or two RMS norms");
    m.def("qkv_rows", &qkv_rows, "query and key row norms, value blend, page write");
    m.def("sigmoid_rows", &sigmoid_rows, "sigmoid attention over pages, row by row");
    m.def("sigmoid_tiles", &sigmoid_tiles, "sigmoid attention over pages, tiles of prompt rows");
}
