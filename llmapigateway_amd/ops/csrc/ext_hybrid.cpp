// Torch extension binding of the hybrid-decoder kernels (see ext.cpp for the
// dense ones). Shapes, strides and dtypes are checked here, on the host: the
// kernels assume them.

#include "bind_shared.h"
#include "bind_checks.h"

void bind_parallel(pybind11::module_& m);  // bind_parallel.cpp
void bind_sigmoid(pybind11::module_& m);   // bind_sigmoid.cpp
void bind_streams(pybind11::module_& m);   // bind_streams.cpp

extern "C" {
hipError_t launch_embed_scaled(float*, void*, int64_t, const int64_t*, const void*, float, int, int, int, int, hipStream_t);
hipError_t launch_stream_norm(void*, int64_t, float*, const void*, int, const float*, const float*, const float*, float, int, int, int, int, int, hipStream_t);
hipError_t launch_latent_rows(void*, void*, int, const void*, const float*, const float*, float, int, int, int, const int64_t*, const float*, const int64_t*, int, int, int, hipStream_t);
hipError_t launch_rotate_pairs(void*, int64_t, int64_t, int, const void*, int64_t, int64_t, int, int, const int64_t*, const float*, int, int, hipStream_t);
hipError_t launch_gated_norm(void*, int64_t, const void*, const void*, int64_t, const float*, float, int, int, int, int, int, int, hipStream_t);
hipError_t launch_causal_conv(void*, const void*, int64_t, const float*, const float*, void*, const int64_t*, const int*, const int*, const int*, int, int, int, int, int, int, hipStream_t);
hipError_t launch_head_linear(void*, int64_t, int64_t, const void*, int64_t, int64_t, const void*, int, int, int, int, int, int, hipStream_t);
hipError_t launch_latent_folded_any(void*, const void*, const void*, const float*, float, const int64_t*, const int*, const int*, int, int, int, int, int, int, int, hipStream_t);
hipError_t launch_latent_folded_mfma(void*, float*, float*, const void*, const void*, const float*, float, const int64_t*, const int*, const int*, int, int, int, int, int, int, int, hipStream_t);
hipError_t launch_latent_unfolded(void*, const void*, const void*, const void*, int64_t, const float*, float, const int*, const int*, const int*, const int*, int, int, int, int, int, int, int, hipStream_t);
hipError_t launch_ssd_scan(void*, const void*, int64_t, const float*, const float*, const float*, const float*, int, int, int, int, float*, const int64_t*, const int*, const int*, const int*, int, int, hipStream_t);
hipError_t launch_mlstm_scan(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, const float*, const float*, float, float, int, int, int, float*, float*, float*, const int64_t*, const int*, const int*, const int*, int, int, hipStream_t);
hipError_t launch_ssd_chunked(void*, const void*, int64_t, const float*, const float*, const float*, const float*, int, int, int, int, int, float*, const int64_t*, const int*, const int*, const int*, const int*, const int*, const int*, int, int, float*, void*, hipStream_t);
hipError_t launch_mlstm_chunked(void*, const void*, int64_t, const void*, int64_t, const void*, int64_t, const float*, const float*, float, float, int, int, int, int, float*, float*, float*, const int64_t*, const int*, const int*, const int*, const int*, const int*, const int*, int, int, float*, void*, float*, float*, hipStream_t);
}

namespace {

void embed_scaled(Tensor x, OptTensor x0, Tensor tokens, Tensor embed, double scale) {
    const bool f32 = is_f32(embed, "embed");
    TORCH_CHECK(embed.dim() == 2 && embed.is_contiguous());
    const int W = embed.size(1), T = tokens.numel();
    f32_ptr(x, (int64_t)T * W, "x");
    bool v = vec8({&x, &embed}, {W});
    if (has(x0)) {
        same_type(*x0, embed, "x0");
        check_rows(*x0, T, W, "x0");
        v = v && vec8({&*x0}, {});
    }
    CHECK_HIP(launch_embed_scaled(x.data_ptr<float>(), has(x0) ? x0->data_ptr() : nullptr,
                                  has(x0) ? x0->stride(0) : 0, i64_ptr(tokens, T, "tokens"),
                                  embed.data_ptr(), (float)scale, T, W, f32, v,
                                  current_stream()));
}

void stream_norm(Tensor& out, Tensor& x, const OptTensor& delta, const OptTensor& vec,
                 const Tensor* w, const Tensor* b, double eps, bool replace) {
    const bool f32 = is_f32(out, "out");
    TORCH_CHECK(x.dim() == 2);
    const int T = x.size(0), W = x.size(1);
    f32_ptr(x, (int64_t)T * W, "x");
    check_rows(out, T, W, "out");
    TORCH_CHECK(!replace || has(delta), "replace needs delta");
    bool v = vec8({&x, &out}, {W}), d32 = false;
    if (has(delta)) {
        check_rows(*delta, T, W, "delta");
        TORCH_CHECK(delta->is_contiguous());
        d32 = is_f32(*delta, "delta");
        TORCH_CHECK(d32 || !f32, "delta: bf16 beside fp32");
        v = v && vec8({&*delta}, {});
    }
    const float* vp = nullptr;
    if (has(vec)) {
        vp = f32_ptr(*vec, W, "vec");
        v = v && vec8({&*vec}, {});
    }
    CHECK_HIP(launch_stream_norm(
        out.data_ptr(), out.stride(0), x.data_ptr<float>(),
        has(delta) ? delta->data_ptr() : nullptr, d32, vp, w ? f32_ptr(*w, W, "w") : nullptr,
        b ? f32_ptr(*b, W, "b") : nullptr, (float)eps, replace, T, W, f32, v,
        current_stream()));
}

void add_layernorm(Tensor out, Tensor x, OptTensor delta, OptTensor vec, Tensor w, Tensor b,
                   double eps, bool replace) {
    stream_norm(out, x, delta, vec, &w, &b, eps, replace);
}

void add_cast(Tensor out, Tensor x, OptTensor delta) {
    stream_norm(out, x, delta, c10::nullopt, nullptr, nullptr, 0.0, false);
}

void latent_rows(Tensor cq, Tensor latent, Tensor d, Tensor q_norm, Tensor kv_norm,
                 double eps, int64_t rot, Tensor positions, Tensor cos_sin,
                 Tensor slot_mapping) {
    const bool f32 = is_f32(d, "d");
    const int64_t qr = q_norm.numel(), rank = kv_norm.numel(), T = d.size(0);
    same_type(d, latent, "latent");
    same_type(d, cq, "cq");
    TORCH_CHECK(d.dim() == 2 && d.is_contiguous() && d.size(1) == qr + rank + rot && rot % 2 == 0);
    TORCH_CHECK(cq.is_contiguous() && cq.numel() == T * qr);
    TORCH_CHECK(latent.dim() == 3 && latent.is_contiguous() && latent.size(2) >= rank + rot);
    TORCH_CHECK(cos_sin.dim() == 2 && cos_sin.size(1) == rot);
    CHECK_HIP(launch_latent_rows(
        cq.data_ptr(), latent.data_ptr(), latent.size(2), d.data_ptr(),
        f32_ptr(q_norm, qr, "q_norm"), f32_ptr(kv_norm, rank, "kv_norm"), (float)eps, qr,
        rank, rot, i64_ptr(positions, T, "positions"),
        f32_ptr(cos_sin, cos_sin.numel(), "cos_sin"), i64_ptr(slot_mapping, T, "slots"), T,
        f32, vec8({&d, &cq, &latent, &q_norm, &kv_norm}, {qr, rank}), current_stream()));
}

void check_heads(const Tensor& t, int64_t T, int64_t H, const char* name) {
    TORCH_CHECK(t.is_cuda() && t.dim() == 3 && t.size(0) == T && t.size(1) == H &&
                (t.stride(2) == 1 || t.size(2) <= 1), name, ": [T, H, dense]");
}

void rotate_pairs(Tensor out, Tensor x, Tensor positions, Tensor cos_sin) {
    const bool f32 = is_f32(x, "x");
    same_type(x, out, "out");
    const int64_t T = x.size(0), H = x.size(1), rot = x.size(2);
    check_heads(x, T, H, "x");
    check_heads(out, T, H, "out");
    TORCH_CHECK(out.size(2) >= rot && cos_sin.dim() == 2 && cos_sin.size(1) == rot);
    CHECK_HIP(launch_rotate_pairs(
        out.data_ptr(), out.stride(0), out.stride(1), out.size(2), x.data_ptr(),
        x.stride(0), x.stride(1), rot, H, i64_ptr(positions, T, "positions"),
        f32_ptr(cos_sin, cos_sin.numel(), "cos_sin"), T, f32, current_stream()));
}

void head_linear(Tensor y, Tensor x, Tensor w) {
    const bool f32 = is_f32(x, "x");
    same_type(x, y, "y");
    same_type(x, w, "w");
    TORCH_CHECK(w.dim() == 3 && w.is_contiguous());
    const int64_t T = x.size(0), H = w.size(0), N = w.size(1), K = w.size(2);
    check_heads(x, T, H, "x");
    check_heads(y, T, H, "y");
    TORCH_CHECK(x.size(2) == K && y.size(2) == N, "head_linear: sizes");
    CHECK_HIP(launch_head_linear(y.data_ptr(), y.stride(0), y.stride(1), x.data_ptr(),
                                 x.stride(0), x.stride(1), w.data_ptr(), T, N, K, H, f32,
                                 vec8({&x, &w}, {K}), current_stream()));
}

void latent_attention_folded(Tensor out, Tensor q, Tensor latent, Tensor sink, double scale,
                             Tensor positions, Tensor row_seg, Tensor tables,
                             int64_t nsplit, OptTensor part_acc, OptTensor part_ml) {
    const bool f32 = is_f32(q, "q");
    same_type(q, latent, "latent");
    same_type(q, out, "out");
    TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && out.dim() == 3 && out.is_contiguous());
    TORCH_CHECK(latent.dim() == 3 && latent.is_contiguous() && latent.size(2) == q.size(2));
    const int64_t T = q.size(0), H = q.size(1), rank = out.size(2);
    TORCH_CHECK(out.size(0) == T && out.size(1) == H && rank <= latent.size(2));
    TORCH_CHECK(tables.dim() == 2);
    if (nsplit > 0) {  // MFMA form
        float *pa = nullptr, *pm = nullptr;
        if (nsplit > 1) {
            TORCH_CHECK(has(part_acc) && has(part_ml));
            TORCH_CHECK(part_acc->numel() >= T * H * nsplit * rank &&
                        part_ml->numel() >= T * H * nsplit * 2, "folded: scratch too small");
            f32_ptr(*part_acc, part_acc->numel(), "part_acc");
            f32_ptr(*part_ml, part_ml->numel(), "part_ml");
            pa = part_acc->data_ptr<float>();
            pm = part_ml->data_ptr<float>();
        }
        TORCH_CHECK(!f32 && vec8({&q, &latent}, {q.size(2)}) && q.size(2) <= 576);
        CHECK_HIP(launch_latent_folded_mfma(
            out.data_ptr(), pa, pm, q.data_ptr(), latent.data_ptr(), f32_ptr(sink, H, "sink"),
            (float)scale, i64_ptr(positions, T, "positions"),
            i32_ptr(row_seg, T, "row_seg"), i32_ptr(tables, 1, "tables"), T, H, rank,
            q.size(2), latent.size(1), tables.size(1), nsplit, current_stream()));
        return;
    }
    CHECK_HIP(launch_latent_folded_any(
        out.data_ptr(), q.data_ptr(), latent.data_ptr(), f32_ptr(sink, H, "sink"),
        (float)scale, i64_ptr(positions, T, "positions"), i32_ptr(row_seg, T, "row_seg"),
        i32_ptr(tables, 1, "tables"), T, H, rank, q.size(2), latent.size(1), tables.size(1),
        f32, current_stream()));
}

void latent_attention_unfolded(Tensor out, Tensor q, Tensor kv, Tensor lat, Tensor sink,
                               double scale, Tensor cu_q, Tensor cu_k, Tensor tile_seg,
                               Tensor tile_off, int64_t tile_rows, int64_t dim, int64_t vdim,
                               int64_t rank) {
    check_bf16(q, "q");
    check_bf16(kv, "kv");
    check_bf16(lat, "lat");
    check_bf16(out, "out");
    TORCH_CHECK(q.dim() == 3 && q.is_contiguous() && out.is_contiguous());
    const int64_t H = q.size(1), rot = q.size(2) - dim, keys = lat.size(0);
    TORCH_CHECK(rot > 0 && out.numel() >= q.size(0) * H * vdim);
    TORCH_CHECK(kv.is_contiguous() && kv.dim() == 2 && kv.size(0) == keys &&
                kv.size(1) == H * (dim + vdim));
    TORCH_CHECK(lat.is_contiguous() && lat.dim() == 2 && lat.size(1) >= rank + rot);
    TORCH_CHECK(vec8({&q, &kv, &lat}, {dim, rot, vdim, rank, lat.size(1)}));
    const int64_t S = cu_q.numel() - 1, nt = tile_seg.numel();
    CHECK_HIP(launch_latent_unfolded(
        out.data_ptr(), q.data_ptr(), kv.data_ptr(), lat.data_ptr(), lat.size(1),
        f32_ptr(sink, H, "sink"), (float)scale, i32_ptr(cu_q, S + 1, "cu_q"),
        i32_ptr(cu_k, S + 1, "cu_k"), i32_ptr(tile_seg, nt, "tile_seg"),
        i32_ptr(tile_off, nt, "tile_off"), nt, tile_rows, H, dim, rot, vdim, rank,
        current_stream()));
}

void causal_conv(Tensor y, Tensor x, Tensor w_t, Tensor b, Tensor state, Tensor positions,
                 Tensor cu, Tensor slots, Tensor row_seg) {
    const bool f32 = is_f32(x, "x");
    same_type(x, y, "y");
    same_type(x, state, "state");
    TORCH_CHECK(w_t.dim() == 2);
    const int64_t T = x.size(0), C = x.size(1), taps = w_t.size(0), S = slots.numel();
    check_rows(x, T, C, "x");
    TORCH_CHECK(y.is_contiguous() && y.numel() == T * C && taps >= 1);
    TORCH_CHECK(state.dim() == 3 && state.is_contiguous() && state.size(1) == taps - 1 &&
                state.size(2) == C);
    CHECK_HIP(launch_causal_conv(
        y.data_ptr(), x.data_ptr(), x.stride(0), f32_ptr(w_t, taps * C, "w_t"),
        f32_ptr(b, C, "b"), state.data_ptr(), i64_ptr(positions, T, "positions"),
        i32_ptr(cu, S + 1, "cu"), i32_ptr(slots, S, "slots"), i32_ptr(row_seg, T, "row_seg"),
        T, S, C, taps, f32, vec8({&x, &y, &w_t, &b, &state}, {C}), current_stream()));
}

const int* seg_list_ptr(const OptTensor& list, int64_t S, int64_t& nseg) {
    nseg = S;
    if (!has(list)) return nullptr;
    nseg = list->numel();
    return i32_ptr(*list, 0, "seg_list");
}

void ssd_scan(Tensor y, Tensor xbc, Tensor dt, Tensor dt_bias, Tensor A_log, Tensor D,
              int64_t H, int64_t P, int64_t N, int64_t G, Tensor state, Tensor positions,
              Tensor cu, Tensor slots, OptTensor seg_list) {
    const bool f32 = is_f32(xbc, "xbc");
    same_type(xbc, y, "y");
    const int64_t T = xbc.size(0), S = slots.numel();
    check_rows(xbc, T, H * P + 2 * G * N, "xbc");
    TORCH_CHECK(G > 0 && H % G == 0 && y.is_contiguous() && y.numel() == T * H * P);
    TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == P && state.size(3) == N);
    TORCH_CHECK(N <= 512, "ssd: state size above 512");
    int64_t nseg;
    const int* list = seg_list_ptr(seg_list, S, nseg);
    f32_ptr(state, state.numel(), "state");
    CHECK_HIP(launch_ssd_scan(
        y.data_ptr(), xbc.data_ptr(), xbc.stride(0), f32_ptr(dt, T * H, "dt"),
        f32_ptr(dt_bias, H, "dt_bias"), f32_ptr(A_log, H, "A_log"), f32_ptr(D, H, "D"), H, P,
        N, G, state.data_ptr<float>(), i64_ptr(positions, T, "positions"),
        i32_ptr(cu, S + 1, "cu"), i32_ptr(slots, S, "slots"), list, nseg, f32,
        current_stream()));
}

void mlstm_scan(Tensor y, Tensor q, Tensor k, Tensor v, Tensor gates, Tensor bias, double cap,
                int64_t H, int64_t dk, int64_t dv, Tensor S, Tensor n, Tensor m,
                Tensor positions, Tensor cu, Tensor slots, OptTensor seg_list) {
    const bool f32 = is_f32(q, "q");
    same_type(q, k, "k");
    same_type(q, v, "v");
    same_type(q, y, "y");
    const int64_t T = q.size(0), ns = slots.numel(), tiles = (dv + 63) / 64;
    check_rows(q, T, H * dk, "q");
    check_rows(k, T, H * dk, "k");
    check_rows(v, T, H * dv, "v");
    TORCH_CHECK(y.is_contiguous() && y.numel() == T * H * dv);
    TORCH_CHECK(S.dim() == 4 && S.size(1) == H && S.size(2) == dv && S.size(3) == dk);
    TORCH_CHECK(dk <= 512, "mlstm: key size above 512");
    const int64_t L = S.size(0);
    f32_ptr(S, S.numel(), "S");
    f32_ptr(n, L * tiles * H * dk, "n");
    f32_ptr(m, L * tiles * H, "m");
    int64_t nseg;
    const int* list = seg_list_ptr(seg_list, ns, nseg);
    CHECK_HIP(launch_mlstm_scan(
        y.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), f32_ptr(gates, T * 2 * H, "gates"), f32_ptr(bias, 2 * H, "bias"),
        (float)cap, 1.0f / std::sqrt((float)dk), H, dk, dv, S.data_ptr<float>(),
        n.data_ptr<float>(), m.data_ptr<float>(), i64_ptr(positions, T, "positions"),
        i32_ptr(cu, ns + 1, "cu"), i32_ptr(slots, ns, "slots"), list, nseg, f32,
        current_stream()));
}

// the chunked forms: segs/first/chunk_seg/chunk_off cut long segments into
// chunks of 64 rows (segment segs[i] has chunks first[i]..first[i+1])
void ssd_chunked(Tensor y, Tensor xbc, Tensor dt, Tensor dt_bias, Tensor A_log, Tensor D,
                 int64_t H, int64_t P, int64_t N, int64_t G, Tensor state, Tensor positions,
                 Tensor cu, Tensor slots, Tensor segs, Tensor first, Tensor chunk_seg,
                 Tensor chunk_off) {
    check_bf16(xbc, "xbc");
    check_bf16(y, "y");
    const int64_t T = xbc.size(0), S = slots.numel();
    const int64_t L = segs.numel(), nc = chunk_seg.numel();
    check_rows(xbc, T, H * P + 2 * G * N, "xbc");
    TORCH_CHECK(G > 0 && H % G == 0 && y.is_contiguous() && y.numel() == T * H * P);
    TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == P && state.size(3) == N);
    TORCH_CHECK(vec8({&xbc}, {P, N}));
    f32_ptr(state, state.numel(), "state");
    const auto dev = xbc.options();
    auto Fb = torch::empty({2, H, T}, dev.dtype(torch::kFloat32));
    auto planes = torch::empty({2, nc, H, P, N}, dev);
    CHECK_HIP(launch_ssd_chunked(
        y.data_ptr(), xbc.data_ptr(), xbc.stride(0), f32_ptr(dt, T * H, "dt"),
        f32_ptr(dt_bias, H, "dt_bias"), f32_ptr(A_log, H, "A_log"), f32_ptr(D, H, "D"), T, H,
        P, N, G, state.data_ptr<float>(), i64_ptr(positions, T, "positions"),
        i32_ptr(cu, S + 1, "cu"), i32_ptr(slots, S, "slots"), i32_ptr(segs, L, "segs"),
        i32_ptr(first, L + 1, "first"), i32_ptr(chunk_seg, nc, "chunk_seg"),
        i32_ptr(chunk_off, nc, "chunk_off"), L, nc, Fb.data_ptr<float>(), planes.data_ptr(),
        current_stream()));
}

void mlstm_chunked(Tensor y, Tensor q, Tensor k, Tensor v, Tensor gates, Tensor bias,
                   double cap, int64_t H, int64_t dk, int64_t dv, Tensor S, Tensor n, Tensor m,
                   Tensor positions, Tensor cu, Tensor slots, Tensor segs, Tensor first,
                   Tensor chunk_seg, Tensor chunk_off) {
    check_bf16(q, "q");
    check_bf16(k, "k");
    check_bf16(v, "v");
    check_bf16(y, "y");
    const int64_t T = q.size(0), ns = slots.numel(), tiles = (dv + 63) / 64;
    const int64_t L = segs.numel(), nc = chunk_seg.numel();
    check_rows(q, T, H * dk, "q");
    check_rows(k, T, H * dk, "k");
    check_rows(v, T, H * dv, "v");
    TORCH_CHECK(y.is_contiguous() && y.numel() == T * H * dv);
    TORCH_CHECK(S.dim() == 4 && S.size(1) == H && S.size(2) == dv && S.size(3) == dk);
    TORCH_CHECK(vec8({&q, &k, &v}, {dk, dv}));
    f32_ptr(S, S.numel(), "S");
    f32_ptr(n, S.size(0) * tiles * H * dk, "n");
    f32_ptr(m, S.size(0) * tiles * H, "m");
    const auto f32 = q.options().dtype(torch::kFloat32);
    auto Fb = torch::empty({2, H, T}, f32);
    auto planes = torch::empty({2, nc, H, dv, dk}, q.options());
    auto n_in = torch::empty({nc, H, dk}, f32);
    auto m_in = torch::empty({nc, H}, f32);
    CHECK_HIP(launch_mlstm_chunked(
        y.data_ptr(), q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(),
        v.stride(0), f32_ptr(gates, T * 2 * H, "gates"), f32_ptr(bias, 2 * H, "bias"),
        (float)cap, 1.0f / std::sqrt((float)dk), T, H, dk, dv, S.data_ptr<float>(),
        n.data_ptr<float>(), m.data_ptr<float>(), i64_ptr(positions, T, "positions"),
        i32_ptr(cu, ns + 1, "cu"), i32_ptr(slots, ns, "slots"), i32_ptr(segs, L, "segs"),
        i32_ptr(first, L + 1, "first"), i32_ptr(chunk_seg, nc, "chunk_seg"),
        i32_ptr(chunk_off, nc, "chunk_off"), L, nc, Fb.data_ptr<float>(), planes.data_ptr(),
        n_in.data_ptr<float>(), m_in.data_ptr<float>(), current_stream()));
}

// mode 0: rms(y) w sigmoid(gate), 1: rms(y silu(gate)) w, 2: rms(y) w silu(gate)
void gated_norm(Tensor out, Tensor y, Tensor gate, Tensor w, int64_t groups, double eps,
                int64_t mode) {
    const bool f32 = is_f32(y, "y");
    same_type(y, gate, "gate");
    same_type(y, out, "out");
    const int64_t T = y.size(0), W = y.size(1);
    TORCH_CHECK(y.is_contiguous());
    check_rows(out, T, W, "out");
    check_rows(gate, T, W, "gate");
    TORCH_CHECK(groups > 0 && W % groups == 0);
    const int64_t gs = W / groups;
    CHECK_HIP(launch_gated_norm(out.data_ptr(), out.stride(0), y.data_ptr(), gate.data_ptr(),
                                gate.stride(0), f32_ptr(w, W, "w"), (float)eps, groups, gs,
                                mode, T, f32, vec8({&out, &y, &gate, &w}, {gs}),
                                current_stream()));
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
    m.def("embed_scaled", &embed_scaled, "scaled embedding into the fp32 stream");
    m.def("add_layernorm", &add_layernorm, "stream add + layer norm");
    m.def("add_cast", &add_cast, "stream add + copy in the compute dtype");
    m.def("latent_rows", &latent_rows, "latent norms + key rotation + page write");
    m.def("rotate_pairs", &rotate_pairs, "interleaved-pair rotation");
    m.def("head_linear", &head_linear, "per-head products");
    m.def("latent_attention_folded", &latent_attention_folded,
          "paged attention in the latent space, with a sink");
    m.def("latent_attention_unfolded", &latent_attention_unfolded,
          "varlen causal attention over per-head keys and values, with a sink");
    m.def("causal_conv", &causal_conv, "segmented causal convolution + silu");
    m.def("ssd_scan", &ssd_scan, "Mamba-2 recurrence, token by token");
    m.def("mlstm_scan", &mlstm_scan, "mLSTM recurrence, token by token");
    m.def("ssd_chunked", &ssd_chunked, "Mamba-2 recurrence, chunked");
    m.def("mlstm_chunked", &mlstm_chunked, "mLSTM recurrence, chunked");
    m.def("gated_norm", &gated_norm, "group RMS norm with a gate");
    bind_parallel(m);
    bind_sigmoid(m);
    bind_streams(m);
    bind_shared(m);
}
