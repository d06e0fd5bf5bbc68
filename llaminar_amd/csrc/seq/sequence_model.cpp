// Steps of a sequence model: buffers, per-sequence state and the order of launches.
// All arithmetic is behind the entry points of seq_api.h and decode_api.h.
#include "llaminar_amd/sequence_model.h"

#include <hip/hip_runtime_api.h>

#include <algorithm>
#include <cstdarg>
#include <cstdio>
#include <cstring>
#include <map>
#include <utility>
#include <vector>

#include "llaminar_amd/decode_api.h"
#include "llaminar_amd/ql_api.h"
#include "llaminar_amd/seq_api.h"

namespace
{
    thread_local char g_error[512] = "";

    bool fail(const char *fn, const char *fmt, ...)
    {
        char msg[400];
        va_list ap;
        va_start(ap, fmt);
        vsnprintf(msg, sizeof msg, fmt, ap);
        va_end(ap);
        snprintf(g_error, sizeof g_error, "[llam_seqm_%s] %s", fn, msg);
        fprintf(stderr, "%s\n", g_error);
        return false;
    }

    // a failed entry point has already printed its reason
    bool forward(const char *fn, bool ok)
    {
        if (!ok)
            snprintf(g_error, sizeof g_error, "[llam_seqm_%s] %s", fn, llam_ql_last_error());
        return ok;
    }

    bool hip_ok(const char *fn, const char *what, hipError_t e)
    {
        return e == hipSuccess || fail(fn, "%s: %s", what, hipGetErrorString(e));
    }

    int pad(int n, int to) { return (n + to - 1) / to * to; }
    int P(int n) { return pad(n, 64); }
    int A(int n) { return n <= 64 ? 64 : n <= 128 ? 128 : 256; } // heads of the grouped-query attention
    bool gated(int ffn) { return ffn == LLAM_FFN_GATED || ffn == LLAM_FFN_GATED_CLAMP; }
    int value_pad(const llam_seqm_layer &w) { return w.mixer == LLAM_MIXER_ATTENTION ? A(w.vdim) : P(w.vdim); }
    // columns of the buffer a mixer writes its heads to: a parallel layer's feed-forward lies behind them
    int mix_columns(const llam_seqm_layer &w) { return w.heads * value_pad(w) + (w.parallel && w.ffn ? P(w.ff) : 0); }

    constexpr int ROW_MAX = 16;         // rows of the row-at-a-time kernels
    constexpr int NORM_FUSE_MAX = 8192; // values a linear layer norms by itself
    constexpr int LOGIT_ROWS = 64;      // rows of logits computed at a time
    constexpr int DECODE_RING = 4096;   // tokens kept on the device between two host reads

    struct Model
    {
        llam_seqm_config cfg{};
        std::vector<llam_seqm_layer> layers;
        std::vector<bool> layer_set;
        llam_seqm_globals globals{};
        bool ready = false;
        hipStream_t stream = nullptr;
        std::vector<void *> owned;
        size_t owned_bytes = 0;
        std::vector<void *> cache;   // per layer: latent cache (its own), else null
        std::vector<void *> values;  // per attention layer: the cache's values (keys in `cache`)
        std::vector<int> cache_rows; // per attention layer: rows of its ring
        std::vector<float *> memory; // per layer: matrix memory, or state of the delta rule
        std::vector<float *> mem_m;  // per layer: running maxima, or recent inputs of the convolution
        int32_t *history = nullptr;  // ids of every slot, where pairs of them are embedded
        size_t slot_bytes = 0;

        int wp = 0, vp = 0, elem = 2;
        float *x = nullptr, *in = nullptr, *z = nullptr, *logits = nullptr, *lat_scratch = nullptr;
        void *h = nullptr, *h2 = nullptr, *q = nullptr, *qlat = nullptr, *olat = nullptr, *mix = nullptr, *act = nullptr;
        void *scratch = nullptr, *arg_scratch = nullptr;
        size_t lat_floats = 0, scratch_bytes = 0;
        // integers of a step: ids, slot and position per row; first row, tokens, slot, position per entry; wanted rows
        int32_t *meta = nullptr, *h_meta = nullptr, *best = nullptr, *ring = nullptr, *count = nullptr;
        float *trace = nullptr;
        struct Graph
        {
            hipGraphExec_t exec = nullptr;
        };
        std::map<std::pair<int, int>, Graph> graphs; // by (sequences, bound on the length)
        hipEvent_t ev[2] = {nullptr, nullptr};

        ~Model()
        {
            (void)hipSetDevice(cfg.device_id);
            if (stream)
                (void)hipStreamSynchronize(stream);
            for (auto &g : graphs)
                if (g.second.exec)
                    (void)hipGraphExecDestroy(g.second.exec);
            for (hipEvent_t e : ev)
                if (e)
                    (void)hipEventDestroy(e);
            for (void *p : owned)
                (void)hipFree(p);
            if (h_meta)
                (void)hipHostFree(h_meta);
            if (stream)
                (void)hipStreamDestroy(stream);
        }

        void *take(const char *fn, size_t bytes)
        {
            void *p = nullptr;
            bytes = std::max<size_t>(bytes, 256);
            hipError_t e = hipMalloc(&p, bytes);
            if (e != hipSuccess)
            {
                fail(fn, "hipMalloc(%zu): %s", bytes, hipGetErrorString(e));
                return nullptr;
            }
            owned.push_back(p);
            owned_bytes += bytes;
            return p;
        }

        int32_t *ids() const { return meta; }
        int32_t *row_slot() const { return meta + cfg.max_rows; }
        int32_t *row_pos() const { return meta + 2 * cfg.max_rows; }
        int32_t *want() const { return meta + 3 * cfg.max_rows; }
        int32_t *entry(int k) const { return meta + 4 * cfg.max_rows + k * cfg.slots; } // row0, ntok, slot, pos
        size_t meta_ints() const { return 4 * (size_t)cfg.max_rows + 4 * (size_t)cfg.slots; }
        llam_seq_entries entries() const { return {entry(0), entry(1), entry(2), entry(3)}; }
    };

    // what a step looks like to the layers: `single` one-token entries first, then the portions
    struct Step
    {
        int M = 0, single = 0;
        int max_len = 1; // bound on the length of the one-token entries' sequences
        std::vector<std::pair<int, int>> portions; // (tokens, length afterwards) of entries single ..
        const int32_t *row_slot = nullptr, *row_pos = nullptr;
    };

    struct Launcher
    {
        Model &md;
        const char *fn;
        const llam_seqm_config &c;
        void *st;

        Launcher(Model &model, const char *name) : md(model), fn(name), c(model.cfg), st(model.stream) {}

        bool linear(const void *a, int lda, const void *w, int N, int K, void *y, int ldy, int out, int M,
                    const float *bias = nullptr, const float *norm = nullptr, int k_real = 0, void *h_out = nullptr,
                    int batch = 1, long as = 0, long ws = 0, long ys = 0, float limit = 0.0f)
        {
            llam_seq_linear_args l{};
            l.limit = limit;
            l.d_a = a, l.lda = lda, l.d_w = w, l.N = N, l.K = K, l.d_y = y, l.ldy = ldy, l.out = out, l.M = M;
            l.d_bias = bias, l.d_norm = norm, l.k_real = k_real, l.eps = c.eps, l.d_h_out = h_out;
            l.batch = batch, l.a_stride = as, l.w_stride = ws, l.y_stride = ys;
            return forward(fn, llam_seq_linear(&l, c.dtype, c.device_id, st));
        }

        static bool fused(int M, int K) { return M <= ROW_MAX && (long)M * K <= NORM_FUSE_MAX; }

        // y = W rms(x) norm: in one launch for a few rows
        bool norm_linear(const float *x, int ldx, const float *norm, int k_real, const void *w, int N, void *y, int ldy,
                         int out, int M, const float *bias = nullptr, bool keep_h = false, float limit = 0.0f)
        {
            const int K = P(k_real);
            if (fused(M, K))
                return linear(x, ldx, w, N, K, y, ldy, out, M, bias, norm, k_real, keep_h ? md.h : nullptr, 1, 0, 0, 0, limit);
            return forward(fn, llam_seq_rmsnorm(x, ldx, nullptr, norm, c.eps, k_real, md.h, M, K, c.dtype, c.device_id, st)) &&
                   linear(md.h, K, w, N, K, y, ldy, out, M, bias, nullptr, 0, nullptr, 1, 0, 0, 0, limit);
        }

        int gated_out(const llam_seqm_layer &w) { return w.ffn == LLAM_FFN_GATED_CLAMP ? LLAM_SEQ_OUT_GATED_CLAMP : LLAM_SEQ_OUT_GATED; }

        // the mixer's projections of x; a parallel layer's gate and up projections go with them
        bool project(const llam_seqm_layer &w, int n_in, const Step &s)
        {
            if (!w.parallel || w.ffn == LLAM_FFN_NONE)
                return norm_linear(md.x, md.wp, w.norm1, c.width, w.w_in, n_in, md.in, n_in, LLAM_SEQ_OUT_F32, s.M);
            const int K = md.wp, fp = P(w.ff), ldm = mix_columns(w);
            llam_seq_linear_args a{}, f{};
            const bool fuse = fused(s.M, K);
            if (!fuse && !forward(fn, llam_seq_rmsnorm_pair(md.x, md.wp, w.norm1, w.norm2, c.eps, c.width, md.h, md.h2, s.M, K, c.dtype, c.device_id, st)))
                return false;
            a.d_a = fuse ? md.x : md.h, a.d_w = w.w_in, a.d_y = md.in, a.N = n_in, a.ldy = n_in, a.out = LLAM_SEQ_OUT_F32;
            f.d_a = fuse ? md.x : md.h2, f.d_w = w.w_up, f.N = 2 * fp, f.ldy = ldm, f.out = gated_out(w), f.limit = w.limit;
            f.d_y = static_cast<char *>(md.mix) + (size_t)(ldm - fp) * md.elem;
            a.d_norm = fuse ? w.norm1 : nullptr, f.d_norm = fuse ? w.norm2 : nullptr;
            for (llam_seq_linear_args *l : {&a, &f})
                l->M = s.M, l->K = K, l->lda = fuse ? md.wp : K, l->k_real = c.width, l->eps = c.eps, l->batch = 1;
            return forward(fn, llam_seq_linear_pair(&a, &f, c.dtype, c.device_id, st));
        }

        // x += W_out of the mixer's heads (and of a parallel layer's feed-forward)
        bool add_output(const llam_seqm_layer &w, const Step &s)
        {
            const int K = mix_columns(w);
            return linear(md.mix, K, w.w_out, md.wp, K, md.x, md.wp, LLAM_SEQ_OUT_ADD, s.M);
        }

        bool attention(const llam_seqm_layer &w, int index, const Step &s)
        {
            const bool own = w.kv_from < 0;
            const int from = own ? index : w.kv_from;
            llam_seq_attention_args a{};
            a.heads = w.heads, a.kv_heads = w.kv_heads, a.dim = A(w.dim), a.vdim = A(w.vdim);
            a.ring = md.cache_rows[from], a.chunk = w.chunk, a.scale = w.scale, a.d_k = md.cache[from], a.d_v = md.values[from];
            const int n_in = w.heads * a.dim + (own ? w.kv_heads * (a.dim + a.vdim) : 0), ldm = mix_columns(w);
            if (!project(w, n_in, s) ||
                !forward(fn, llam_seq_rotary(&a, md.in, n_in, own, w.turns, w.rot_dims, s.row_slot, s.row_pos, md.q, s.M, c.dtype, c.device_id, st)))
                return false;
            const llam_seq_entries e = md.entries();
            if (s.single && !forward(fn, llam_seq_attention(&a, md.q, &e, 0, s.single, 1, s.max_len, md.mix, ldm, md.lat_scratch, md.lat_floats,
                                                            c.dtype, c.device_id, st)))
                return false;
            for (size_t k = 0; k < s.portions.size(); ++k)
                if (!forward(fn, llam_seq_attention(&a, md.q, &e, s.single + (int)k, 1, s.portions[k].first, s.portions[k].second, md.mix, ldm,
                                                    md.lat_scratch, md.lat_floats, c.dtype, c.device_id, st)))
                    return false;
            return add_output(w, s);
        }

        bool delta(const llam_seqm_layer &w, int index, const Step &s)
        {
            const int H = w.heads, G = w.kv_heads, dp = P(w.dim), vp = P(w.vdim);
            const int n_in = pad(2 * G * dp + 2 * H * vp + 2 * H, 16);
            if (!project(w, n_in, s))
                return false;
            llam_seq_delta_args a{};
            a.d_proj = md.in, a.ldp = n_in, a.d_conv = w.conv, a.d_a_log = w.a_log, a.d_dt_bias = w.dt_bias, a.d_norm = w.head_norm;
            a.d_state = md.memory[index], a.d_recent = md.mem_m[index], a.d_y = md.mix, a.ldy = mix_columns(w);
            a.heads = H, a.kv_heads = G, a.dim = dp, a.vdim = vp, a.dim_real = w.dim, a.vdim_real = w.vdim, a.taps = w.taps, a.eps = c.eps;
            const llam_seq_entries e = md.entries();
            if (s.single && !forward(fn, llam_seq_delta_decode(&a, &e, 0, s.single, c.dtype, c.device_id, st)))
                return false;
            for (size_t k = 0; k < s.portions.size(); ++k)
                if (!forward(fn, llam_seq_delta_prefill(&a, &e, s.single + (int)k, s.portions[k].first, md.scratch, md.scratch_bytes, c.dtype,
                                                        c.device_id, st)))
                    return false;
            return add_output(w, s);
        }

        bool latent(const llam_seqm_layer &w, int index, const Step &s)
        {
            const int H = w.heads, dp = P(w.dim), vp = P(w.vdim), qp = P(w.q_rank), rp = P(w.kv_rank);
            const bool own = w.kv_from < 0;
            const int n_in = qp + (own ? rp : 0);
            if (!project(w, n_in, s))
                return false;
            void *cache = md.cache[own ? index : w.kv_from];
            if (own && !forward(fn, llam_seq_latent_append(md.in + qp, n_in, w.kv_norm, c.eps, w.kv_rank, s.row_slot, s.row_pos,
                                                           cache, s.M, rp, c.cap, c.dtype, c.device_id, st)))
                return false;
            if (!norm_linear(md.in, n_in, w.q_norm, w.q_rank, w.w_uq, H * dp, md.q, H * dp, LLAM_SEQ_OUT_ELEM, s.M) ||
                !linear(md.q, H * dp, w.w_uk_t, rp, dp, md.qlat, H * rp, LLAM_SEQ_OUT_ELEM, s.M, nullptr, nullptr, 0, nullptr, H,
                        dp, (long)rp * dp, rp))
                return false;
            const llam_seq_entries e = md.entries();
            if (s.single && !forward(fn, llam_seq_latent_attention(md.qlat, cache, &e, 0, s.single, 1, s.max_len, H, rp, c.cap, w.scale,
                                                                   md.olat, md.lat_scratch, md.lat_floats, c.dtype, c.device_id, st)))
                return false;
            for (size_t k = 0; k < s.portions.size(); ++k)
                if (!forward(fn, llam_seq_latent_attention(md.qlat, cache, &e, s.single + (int)k, 1, s.portions[k].first,
                                                           s.portions[k].second, H, rp, c.cap, w.scale, md.olat, md.lat_scratch,
                                                           md.lat_floats, c.dtype, c.device_id, st)))
                    return false;
            return linear(md.olat, H * rp, w.w_uv, vp, rp, md.mix, mix_columns(w), LLAM_SEQ_OUT_ELEM, s.M, nullptr, nullptr, 0, nullptr, H,
                          rp, (long)vp * rp, vp) &&
                   add_output(w, s);
        }

        bool memory(const llam_seqm_layer &w, int index, const Step &s)
        {
            const int H = w.heads, dp = P(w.dim), vp = P(w.vdim);
            const int n_in = pad(2 * H * (dp + vp) + 2 * H, 16);
            if (!project(w, n_in, s))
                return false;
            llam_seq_memory_args a{};
            a.d_proj = md.in, a.ldp = n_in, a.d_gate_bias = w.gate_bias, a.d_norm = w.head_norm;
            a.d_state = md.memory[index], a.d_m = md.mem_m[index], a.d_y = md.mix, a.ldy = mix_columns(w);
            a.heads = H, a.dim = dp, a.vdim = vp, a.vdim_real = w.vdim;
            a.q_scale = w.scale, a.gate_cap = w.gate_cap, a.eps = c.eps;
            const llam_seq_entries e = md.entries();
            if (s.single && !forward(fn, llam_seq_memory_decode(&a, &e, 0, s.single, md.scratch, md.scratch_bytes, c.dtype, c.device_id, st)))
                return false;
            for (size_t k = 0; k < s.portions.size(); ++k)
                if (!forward(fn, llam_seq_memory_prefill(&a, &e, s.single + (int)k, s.portions[k].first, md.scratch, md.scratch_bytes,
                                                         c.dtype, c.device_id, st)))
                    return false;
            return add_output(w, s);
        }

        bool ffn(const llam_seqm_layer &w, const Step &s)
        {
            const int fp = P(w.ff), wp = md.wp;
            if (gated(w.ffn))
                return norm_linear(md.x, wp, w.norm2, c.width, w.w_up, 2 * fp, md.act, fp, gated_out(w), s.M, nullptr, false, w.limit) &&
                       linear(md.act, fp, w.w_down, wp, fp, md.x, wp, LLAM_SEQ_OUT_ADD, s.M);
            const int zp = pad(w.experts + (w.shared_ff ? 1 : 0), 16), sp = w.shared_ff ? P(w.shared_ff) : 0;
            if (!norm_linear(md.x, wp, w.norm2, c.width, w.w_router, zp, md.z, zp, LLAM_SEQ_OUT_F32, s.M, w.router_bias, true))
                return false;
            llam_seq_experts_args a{};
            a.d_logits = md.z, a.ldz = zp, a.d_up = w.w_up, a.d_down = w.w_down;
            a.d_shared_up = w.w_shared_up, a.d_shared_down = w.w_shared_down;
            a.up_stride = (long)fp * wp, a.down_stride = (long)wp * fp;
            a.experts = w.experts, a.top = w.top, a.ff = fp, a.shared_ff = sp, a.K = wp, a.N = wp;
            a.d_h = md.h, a.d_x = md.x, a.ldx = wp;
            return forward(fn, llam_seq_experts(&a, s.M, md.scratch, md.scratch_bytes, c.dtype, c.device_id, st));
        }

        bool layers(const Step &s)
        {
            const llam_seqm_globals &gl = md.globals;
            llam_seq_embed_args em{};
            em.d_table = gl.embed, em.vocab = c.vocab, em.width = c.width, em.scale = gl.embed_scale;
            em.d_pairs = gl.pairs, em.buckets = gl.buckets, em.mul_prev = gl.mul_prev, em.mul_cur = gl.mul_cur;
            em.d_row_slot = s.row_slot, em.d_row_pos = s.row_pos, em.d_history = md.history, em.cap = c.cap;
            if (!forward(fn, llam_seq_embed(&em, md.ids(), md.x, s.M, md.wp, c.device_id, st)))
                return false;
            for (int l = 0; l < c.n_layers; ++l)
            {
                const llam_seqm_layer &w = md.layers[l];
                if (!(w.mixer == LLAM_MIXER_LATENT_ATTENTION ? latent(w, l, s) : w.mixer == LLAM_MIXER_MATRIX_MEMORY ? memory(w, l, s)
                      : w.mixer == LLAM_MIXER_ATTENTION ? attention(w, l, s) : delta(w, l, s)))
                    return false;
                if (w.ffn != LLAM_FFN_NONE && !w.parallel && !ffn(w, s))
                    return false;
                if (md.trace && !hip_ok(fn, "hipMemcpy2DAsync", hipMemcpy2DAsync(md.trace + (size_t)l * s.M * c.width, (size_t)c.width * 4, md.x,
                                                                                 (size_t)md.wp * 4, (size_t)c.width * 4, s.M,
                                                                                 hipMemcpyDeviceToHost, md.stream)))
                    return false;
            }
            return true;
        }

        // logits of rows[0 .. n) of the residual stream (nullptr: rows 0 .. n - 1), n <= LOGIT_ROWS
        bool logits(const int32_t *rows, int n)
        {
            if (!rows && fused(n, md.wp))
                return linear(md.x, md.wp, md.globals.head, md.vp, md.wp, md.logits, md.vp, LLAM_SEQ_OUT_F32, n, nullptr,
                              md.globals.final_norm, c.width);
            return forward(fn, llam_seq_rmsnorm(md.x, md.wp, rows, md.globals.final_norm, c.eps, c.width, md.h, n, md.wp, c.dtype,
                                                c.device_id, st)) &&
                   linear(md.h, md.wp, md.globals.head, md.vp, md.wp, md.logits, md.vp, LLAM_SEQ_OUT_F32, n);
        }

        // one greedy step of n sequences, all of it on the device
        bool decode_step(int n, int max_len)
        {
            Step s;
            s.M = s.single = n;
            s.max_len = max_len;
            s.row_slot = md.entry(2);
            s.row_pos = md.entry(3);
            return layers(s) && logits(nullptr, n) &&
                   forward(fn, llam_dec_argmax(md.logits, md.vp, c.vocab, n, md.ids(), md.entry(3), md.arg_scratch, c.device_id, st)) &&
                   forward(fn, llam_seq_record(md.ids(), n, md.ring, md.count, DECODE_RING / n, c.device_id, st));
        }
    };

    bool check_entry(const char *fn, const Model &md, int slot, int pos, int ntok)
    {
        if (slot < 0 || slot >= md.cfg.slots)
            return fail(fn, "slot %d outside [0, %d)", slot, md.cfg.slots);
        if (pos < 0 || ntok < 1 || pos > md.cfg.cap - ntok)
            return fail(fn, "%d tokens at position %d do not fit the %d positions of a slot", ntok, pos, md.cfg.cap);
        return true;
    }
} // namespace

extern "C" const char *llam_seqm_last_error(void) { return g_error; }

extern "C" void *llam_seqm_create(const llam_seqm_config *cfg)
{
    static const char *fn = "create";
    if (!cfg || cfg->width < 1 || cfg->vocab < 1 || cfg->n_layers < 1 || cfg->slots < 1 || cfg->cap < 1 || cfg->max_rows < 1 ||
        cfg->max_rows > 32768 || cfg->slots > 4096)
    {
        fail(fn, "bad configuration");
        return nullptr;
    }
    if (cfg->dtype != LLAM_SEQ_BF16 && cfg->dtype != LLAM_SEQ_F32)
    {
        fail(fn, "dtype %d", cfg->dtype);
        return nullptr;
    }
    int devices = 0;
    if (hipGetDeviceCount(&devices) != hipSuccess || cfg->device_id < 0 || cfg->device_id >= devices)
    {
        fail(fn, "no HIP device %d", cfg->device_id);
        return nullptr;
    }
    Model *md = new Model;
    md->cfg = *cfg;
    md->layers.resize(cfg->n_layers);
    md->layer_set.assign(cfg->n_layers, false);
    md->wp = P(cfg->width);
    md->vp = pad(cfg->vocab, 16);
    md->elem = cfg->dtype == LLAM_SEQ_F32 ? 4 : 2;
    if (!hip_ok(fn, "hipSetDevice", hipSetDevice(cfg->device_id)) ||
        !hip_ok(fn, "hipStreamCreate", hipStreamCreateWithFlags(&md->stream, hipStreamNonBlocking)) ||
        !hip_ok(fn, "hipEventCreate", hipEventCreate(&md->ev[0])) || !hip_ok(fn, "hipEventCreate", hipEventCreate(&md->ev[1])))
    {
        delete md;
        return nullptr;
    }
    return md;
}

extern "C" void llam_seqm_destroy(void *model) { delete static_cast<Model *>(model); }

extern "C" void *llam_seqm_upload(void *model, const void *h_data, size_t bytes)
{
    static const char *fn = "upload";
    Model *md = static_cast<Model *>(model);
    if (!md || !h_data || !hip_ok(fn, "hipSetDevice", hipSetDevice(md->cfg.device_id)))
        return nullptr;
    void *p = md->take(fn, bytes);
    if (p && !hip_ok(fn, "hipMemcpy", hipMemcpy(p, h_data, bytes, hipMemcpyHostToDevice)))
        return nullptr;
    return p;
}

extern "C" bool llam_seqm_set_layer(void *model, int layer, const llam_seqm_layer *w)
{
    static const char *fn = "set_layer";
    Model *md = static_cast<Model *>(model);
    if (!md || !w || layer < 0 || layer >= md->cfg.n_layers)
        return fail(fn, "bad arguments (layer %d)", layer);
    if (w->heads < 1 || w->dim < 1 || w->vdim < 1 || !w->norm1 || !w->w_in || !w->w_out)
        return fail(fn, "layer %d: sizes or tensors of the mixer are missing", layer);
    if (w->mixer == LLAM_MIXER_LATENT_ATTENTION)
    {
        if (w->q_rank < 1 || w->kv_rank < 1 || !w->q_norm || !w->w_uq || !w->w_uk_t || !w->w_uv)
            return fail(fn, "layer %d: sizes or tensors of the latent attention are missing", layer);
        if (w->kv_from < 0)
        {
            if (!w->kv_norm)
                return fail(fn, "layer %d: kv_norm is missing", layer);
        }
        else
        {
            if (w->kv_from >= layer || !md->layer_set[w->kv_from])
                return fail(fn, "layer %d: kv_from %d is not an earlier layer", layer, w->kv_from);
            const llam_seqm_layer &from = md->layers[w->kv_from];
            if (from.mixer != LLAM_MIXER_LATENT_ATTENTION || from.kv_from >= 0 || from.kv_rank != w->kv_rank)
                return fail(fn, "layer %d: layer %d has no latent of its own of rank %d", layer, w->kv_from, w->kv_rank);
        }
    }
    else if (w->mixer == LLAM_MIXER_MATRIX_MEMORY)
    {
        if (!w->gate_bias || !w->head_norm || !(w->gate_cap > 0.0f) || P(w->dim) > 512)
            return fail(fn, "layer %d: tensors of the matrix memory are missing, or dim=%d above 512", layer, w->dim);
    }
    else if (w->mixer == LLAM_MIXER_ATTENTION)
    {
        if (w->kv_heads < 1 || (w->heads % w->kv_heads) != 0 || w->dim > 256 || w->vdim > 256)
            return fail(fn, "layer %d: heads=%d must be a multiple of kv_heads=%d, dim=%d and vdim=%d at most 256", layer, w->heads, w->kv_heads, w->dim, w->vdim);
        if (w->rot_dims < 0 || (w->rot_dims % 2) != 0 || w->rot_dims > w->dim || (w->rot_dims && !w->turns) || w->chunk < 0)
            return fail(fn, "layer %d: rot_dims=%d chunk=%d", layer, w->rot_dims, w->chunk);
        if (w->kv_from >= 0)
        {
            if (w->kv_from >= layer || !md->layer_set[w->kv_from])
                return fail(fn, "layer %d: kv_from %d is not an earlier layer", layer, w->kv_from);
            const llam_seqm_layer &from = md->layers[w->kv_from];
            if (from.mixer != LLAM_MIXER_ATTENTION || from.kv_from >= 0 || from.kv_heads != w->kv_heads || from.dim != w->dim || from.vdim != w->vdim)
                return fail(fn, "layer %d: layer %d has no keys and values of its own of these sizes", layer, w->kv_from);
        }
    }
    else if (w->mixer == LLAM_MIXER_DELTA)
    {
        if (w->kv_heads < 1 || (w->heads % w->kv_heads) != 0 || w->dim > 256 || w->vdim > 4096 || w->taps < 1 || w->taps > 1024)
            return fail(fn, "layer %d: heads=%d must be a multiple of kv_heads=%d, dim=%d at most 256, vdim=%d at most 4096, taps=%d", layer, w->heads, w->kv_heads, w->dim, w->vdim, w->taps);
        if (!w->conv || !w->a_log || !w->dt_bias || !w->head_norm)
            return fail(fn, "layer %d: tensors of the delta rule are missing", layer);
    }
    else
        return fail(fn, "layer %d: mixer kind %d", layer, w->mixer);
    if (w->ffn != LLAM_FFN_NONE)
    {
        if (!gated(w->ffn) && w->ffn != LLAM_FFN_EXPERTS)
            return fail(fn, "layer %d: feed-forward kind %d", layer, w->ffn);
        if (w->parallel && !gated(w->ffn))
            return fail(fn, "layer %d: a parallel layer takes a gated feed-forward", layer);
        if (w->ff < 1 || !w->norm2 || !w->w_up || (!w->w_down && !w->parallel))
            return fail(fn, "layer %d: sizes or tensors of the feed-forward are missing", layer);
        if (w->ffn == LLAM_FFN_EXPERTS &&
            (w->experts < 1 || w->experts > 1024 || w->top < 1 || w->top > w->experts || w->top > 64 || w->shared_ff < 0 || !w->w_router || !w->router_bias ||
             (w->shared_ff && (!w->w_shared_up || !w->w_shared_down))))
            return fail(fn, "layer %d: sizes (experts=%d top=%d) or tensors of the experts", layer, w->experts, w->top);
    }
    md->layers[layer] = *w;
    md->layer_set[layer] = true;
    return true;
}

extern "C" bool llam_seqm_set_globals(void *model, const llam_seqm_globals *g)
{
    static const char *fn = "set_globals";
    Model *md = static_cast<Model *>(model);
    if (!md || !g || !g->embed || !g->final_norm || !g->head || md->ready || (g->pairs && g->buckets < 1))
        return fail(fn, "bad arguments");
    for (int l = 0; l < md->cfg.n_layers; ++l)
        if (!md->layer_set[l])
            return fail(fn, "layer %d is not set", l);
    const llam_seqm_config &c = md->cfg;
    if (!hip_ok(fn, "hipSetDevice", hipSetDevice(c.device_id)))
        return false;
    md->globals = *g;
    const size_t M = c.max_rows, elem = md->elem;
    bool parallel = false;
    size_t n_in = 0, q = 0, lat = 0, mix = 0, act = 0, z = 16, h = md->wp, latf = 0, scratch = 0;
    for (const llam_seqm_layer &w : md->layers)
    {
        const size_t H = w.heads, dp = P(w.dim), vp = P(w.vdim);
        mix = std::max(mix, (size_t)mix_columns(w));
        parallel |= w.parallel && w.ffn;
        if (w.mixer == LLAM_MIXER_LATENT_ATTENTION)
        {
            const size_t rp = P(w.kv_rank);
            n_in = std::max(n_in, (size_t)P(w.q_rank) + rp);
            h = std::max(h, (size_t)P(w.q_rank));
            q = std::max(q, H * dp);
            lat = std::max(lat, H * rp);
            latf = std::max(latf, llam_seq_latent_scratch_floats(c.max_rows, c.slots, w.heads, (int)rp, c.cap));
        }
        else if (w.mixer == LLAM_MIXER_ATTENTION)
        {
            n_in = std::max(n_in, H * A(w.dim) + (w.kv_from < 0 ? (size_t)w.kv_heads * (A(w.dim) + A(w.vdim)) : 0));
            q = std::max(q, H * A(w.dim));
            latf = std::max(latf, llam_seq_attention_scratch_floats(A(w.vdim)));
        }
        else if (w.mixer == LLAM_MIXER_DELTA)
        {
            n_in = std::max(n_in, (size_t)pad((int)(2 * w.kv_heads * dp + 2 * H * vp + 2 * H), 16));
            scratch = std::max(scratch, llam_seq_delta_scratch_bytes(c.max_rows, w.heads, w.kv_heads, (int)dp, (int)vp));
        }
        else
        {
            n_in = std::max(n_in, (size_t)pad((int)(2 * H * (dp + vp) + 2 * H), 16));
            scratch = std::max(scratch, llam_seq_memory_scratch_bytes(std::max(c.max_rows, c.slots), w.heads, (int)dp, (int)vp));
        }
        if (gated(w.ffn) && !w.parallel)
            act = std::max(act, (size_t)P(w.ff));
        if (w.ffn == LLAM_FFN_EXPERTS)
        {
            z = std::max(z, (size_t)pad(w.experts + 1, 16));
            scratch = std::max(scratch, llam_seq_experts_scratch_bytes(c.max_rows, w.experts, w.top, P(w.ff),
                                                                       w.shared_ff ? P(w.shared_ff) : 0, md->wp));
        }
    }
    md->lat_floats = latf;
    md->scratch_bytes = scratch;
    bool ok = (md->x = (float *)md->take(fn, M * md->wp * 4)) && (md->h = md->take(fn, M * h * elem)) && (md->h2 = md->take(fn, parallel ? M * md->wp * elem : 0)) &&
              (md->in = (float *)md->take(fn, M * n_in * 4)) && (md->q = md->take(fn, M * q * elem)) &&
              (md->qlat = md->take(fn, M * lat * elem)) && (md->olat = md->take(fn, M * lat * elem)) &&
              (md->mix = md->take(fn, M * mix * elem)) && (md->act = md->take(fn, M * act * elem)) &&
              (md->z = (float *)md->take(fn, M * z * 4)) && (md->scratch = md->take(fn, scratch)) &&
              (md->lat_scratch = (float *)md->take(fn, latf * 4)) &&
              (md->logits = (float *)md->take(fn, (size_t)std::max(LOGIT_ROWS, c.slots) * md->vp * 4)) &&
              (md->arg_scratch = md->take(fn, llam_dec_argmax_scratch_bytes(std::max(LOGIT_ROWS, c.slots), c.vocab))) &&
              (md->meta = (int32_t *)md->take(fn, md->meta_ints() * 4)) &&
              (md->best = (int32_t *)md->take(fn, (size_t)LOGIT_ROWS * 4)) &&
              (md->ring = (int32_t *)md->take(fn, (size_t)(DECODE_RING + c.slots) * 4)) && (md->count = (int32_t *)md->take(fn, 4));
    if (!ok || !hip_ok(fn, "hipHostMalloc", hipHostMalloc((void **)&md->h_meta, md->meta_ints() * 4, hipHostMallocDefault)))
        return false;
    md->cache.assign(c.n_layers, nullptr);
    md->memory.assign(c.n_layers, nullptr);
    md->mem_m.assign(c.n_layers, nullptr);
    md->values.assign(c.n_layers, nullptr);
    md->cache_rows.assign(c.n_layers, 0);
    if (g->pairs)
    {
        if (!(md->history = (int32_t *)md->take(fn, (size_t)c.slots * c.cap * 4)))
            return false;
        md->slot_bytes += (size_t)c.cap * 4;
    }
    // rows an attention cache must keep: what the widest mask of its readers shows the first token of a step, and the step
    for (int l = 0; l < c.n_layers; ++l)
    {
        const llam_seqm_layer &w = md->layers[l];
        if (w.mixer != LLAM_MIXER_ATTENTION)
            continue;
        const long sight = w.chunk > 0 ? std::min<long>(c.cap, (long)w.chunk - 1 + c.max_rows) : c.cap;
        int &ring = md->cache_rows[w.kv_from >= 0 ? w.kv_from : l];
        ring = std::max(ring, pad((int)sight, 128));
    }
    for (int l = 0; l < c.n_layers; ++l)
    {
        const llam_seqm_layer &w = md->layers[l];
        if (w.mixer == LLAM_MIXER_LATENT_ATTENTION)
        {
            if (w.kv_from >= 0)
                continue;
            const size_t per = (size_t)c.cap * P(w.kv_rank) * elem;
            if (!(md->cache[l] = md->take(fn, per * c.slots)))
                return false;
            md->slot_bytes += per;
        }
        else if (w.mixer == LLAM_MIXER_ATTENTION)
        {
            if (w.kv_from >= 0)
                continue;
            const size_t rows = (size_t)w.kv_heads * md->cache_rows[l], k = rows * A(w.dim) * elem, v = rows * A(w.vdim) * elem;
            if (!(md->cache[l] = md->take(fn, k * c.slots)) || !(md->values[l] = md->take(fn, v * c.slots)))
                return false;
            md->slot_bytes += k + v;
        }
        else if (w.mixer == LLAM_MIXER_DELTA)
        {
            const size_t state = (size_t)w.heads * P(w.dim) * P(w.vdim);
            const size_t recent = (size_t)w.taps * (2 * w.kv_heads * P(w.dim) + w.heads * P(w.vdim));
            if (!(md->memory[l] = (float *)md->take(fn, state * c.slots * 4)) || !(md->mem_m[l] = (float *)md->take(fn, recent * c.slots * 4)))
                return false;
            md->slot_bytes += (state + recent) * 4;
        }
        else
        {
            const size_t per = (size_t)w.heads * P(w.dim) * (P(w.vdim) + 16);
            if (!(md->memory[l] = (float *)md->take(fn, per * c.slots * 4)) ||
                !(md->mem_m[l] = (float *)md->take(fn, (size_t)w.heads * c.slots * 4)))
                return false;
            md->slot_bytes += (per + w.heads) * 4;
        }
    }
    if (!hip_ok(fn, "hipDeviceSynchronize", hipDeviceSynchronize()))
        return false;
    md->ready = true;
    return true;
}

extern "C" bool llam_seqm_forward(void *model, int n, const int32_t *h_slot, const int32_t *h_pos, const int32_t *h_ntok,
                                  const int32_t *h_ids, int n_want, const int32_t *h_want, float *h_logits, int32_t *h_best)
{
    static const char *fn = "forward";
    Model *md = static_cast<Model *>(model);
    if (!md || !md->ready)
        return fail(fn, "the model is not complete");
    const llam_seqm_config &c = md->cfg;
    if (n < 1 || n > c.slots || !h_slot || !h_pos || !h_ntok || !h_ids || n_want < 0 || (n_want && !h_want))
        return fail(fn, "bad arguments (n=%d n_want=%d)", n, n_want);
    if (!hip_ok(fn, "hipSetDevice", hipSetDevice(c.device_id)))
        return false;
    Step s;
    long rows = 0;
    std::vector<bool> seen(c.slots, false);
    for (int e = 0; e < n; ++e)
    {
        if (!check_entry(fn, *md, h_slot[e], h_pos[e], h_ntok[e]))
            return false;
        if (seen[h_slot[e]])
            return fail(fn, "slot %d appears twice", h_slot[e]);
        seen[h_slot[e]] = true;
        rows += h_ntok[e];
    }
    if (rows > c.max_rows)
        return fail(fn, "%ld tokens in a step, at most %d", rows, c.max_rows);
    s.M = (int)rows;
    for (int k = 0; k < n_want; ++k)
        if (h_want[k] < 0 || h_want[k] >= s.M)
            return fail(fn, "wanted row %d outside the step", h_want[k]);
    int32_t *hm = md->h_meta;
    const int R = c.max_rows;
    memcpy(hm, h_ids, sizeof(int32_t) * s.M);
    int at = 0, placed = 0;
    std::vector<int> row0(n);
    for (int e = 0; e < n; ++e)
    {
        row0[e] = at;
        for (int t = 0; t < h_ntok[e]; ++t, ++at)
        {
            hm[R + at] = h_slot[e];
            hm[2 * R + at] = h_pos[e] + t;
        }
    }
    auto place = [&](int e) {
        int32_t *q = hm + 4 * R;
        q[placed] = row0[e];
        q[c.slots + placed] = h_ntok[e];
        q[2 * c.slots + placed] = h_slot[e];
        q[3 * c.slots + placed] = h_pos[e];
        ++placed;
    };
    for (int e = 0; e < n; ++e)
        if (h_ntok[e] == 1)
        {
            place(e);
            s.max_len = std::max(s.max_len, h_pos[e] + 1);
        }
    s.single = placed;
    for (int e = 0; e < n; ++e)
        if (h_ntok[e] > 1)
        {
            place(e);
            s.portions.emplace_back(h_ntok[e], h_pos[e] + h_ntok[e]);
        }
    s.row_slot = md->row_slot();
    s.row_pos = md->row_pos();
    if (!hip_ok(fn, "hipMemcpyAsync", hipMemcpyAsync(md->meta, hm, md->meta_ints() * 4, hipMemcpyHostToDevice, md->stream)))
        return false;
    Launcher run(*md, fn);
    if (!run.layers(s))
        return false;
    for (int w0 = 0; w0 < n_want; w0 += LOGIT_ROWS)
    {
        const int k = std::min(LOGIT_ROWS, n_want - w0);
        if (!hip_ok(fn, "hipMemcpyAsync", hipMemcpyAsync(md->want(), h_want + w0, (size_t)k * 4, hipMemcpyHostToDevice, md->stream)) ||
            !run.logits(md->want(), k))
            return false;
        if (h_logits && !hip_ok(fn, "hipMemcpy2DAsync", hipMemcpy2DAsync(h_logits + (size_t)w0 * c.vocab, (size_t)c.vocab * 4, md->logits,
                                                                         (size_t)md->vp * 4, (size_t)c.vocab * 4, k,
                                                                         hipMemcpyDeviceToHost, md->stream)))
            return false;
        if (h_best && (!forward(fn, llam_dec_argmax(md->logits, md->vp, c.vocab, k, md->best, nullptr, md->arg_scratch, c.device_id, md->stream)) ||
                       !hip_ok(fn, "hipMemcpyAsync", hipMemcpyAsync(h_best + w0, md->best, (size_t)k * 4, hipMemcpyDeviceToHost, md->stream))))
            return false;
        if (!hip_ok(fn, "hipStreamSynchronize", hipStreamSynchronize(md->stream)))
            return false;
    }
    return hip_ok(fn, "hipStreamSynchronize", hipStreamSynchronize(md->stream));
}

extern "C" bool llam_seqm_decode(void *model, int n, const int32_t *h_slot, const int32_t *h_pos, const int32_t *h_ids,
                                 int steps, int32_t *h_out, float *h_ms)
{
    static const char *fn = "decode";
    Model *md = static_cast<Model *>(model);
    if (!md || !md->ready)
        return fail(fn, "the model is not complete");
    const llam_seqm_config &c = md->cfg;
    if (n < 1 || n > c.slots || n > c.max_rows || steps < 1 || !h_slot || !h_pos || !h_ids || !h_out)
        return fail(fn, "bad arguments (n=%d steps=%d)", n, steps);
    if (steps > DECODE_RING / n)
        return fail(fn, "%d steps of %d sequences at a time, at most %d", steps, n, DECODE_RING / n);
    if (!hip_ok(fn, "hipSetDevice", hipSetDevice(c.device_id)))
        return false;
    int len = 0;
    std::vector<bool> seen(c.slots, false);
    int32_t *hm = md->h_meta;
    for (int b = 0; b < n; ++b)
    {
        if (!check_entry(fn, *md, h_slot[b], h_pos[b], steps))
            return false;
        if (seen[h_slot[b]])
            return fail(fn, "slot %d appears twice", h_slot[b]);
        seen[h_slot[b]] = true;
        len = std::max(len, h_pos[b] + steps);
        hm[b] = h_ids[b];
        int32_t *q = hm + 4 * c.max_rows;
        q[b] = b;
        q[c.slots + b] = 1;
        q[2 * c.slots + b] = h_slot[b];
        q[3 * c.slots + b] = h_pos[b];
    }
    int bound = 256; // graphs are kept by powers of two of the length
    while (bound < len)
        bound *= 2;
    bound = std::min(bound, c.cap);
    const int32_t zero = 0;
    if (!hip_ok(fn, "hipMemcpyAsync", hipMemcpyAsync(md->meta, hm, md->meta_ints() * 4, hipMemcpyHostToDevice, md->stream)) ||
        !hip_ok(fn, "hipMemcpyAsync", hipMemcpyAsync(md->count, &zero, 4, hipMemcpyHostToDevice, md->stream)) ||
        !hip_ok(fn, "hipStreamSynchronize", hipStreamSynchronize(md->stream)))
        return false;
    Launcher run(*md, fn);
    int done = 0;
    Model::Graph &g = md->graphs[{n, bound}];
    if (!g.exec)
    {
        // the first step of this shape runs as it is (kernels are loaded then), the others as its graph
        if (!run.decode_step(n, bound) || !hip_ok(fn, "hipStreamSynchronize", hipStreamSynchronize(md->stream)))
            return false;
        done = 1;
        if (steps > 1)
        {
            if (!hip_ok(fn, "hipStreamBeginCapture", hipStreamBeginCapture(md->stream, hipStreamCaptureModeThreadLocal)))
                return false;
            const bool ok = run.decode_step(n, bound);
            hipGraph_t graph = nullptr;
            const hipError_t e = hipStreamEndCapture(md->stream, &graph);
            if (!ok || !hip_ok(fn, "hipStreamEndCapture", e))
                return false;
            const hipError_t ei = hipGraphInstantiate(&g.exec, graph, nullptr, nullptr, 0);
            (void)hipGraphDestroy(graph);
            if (ei != hipSuccess)
            {
                g.exec = nullptr;
                return hip_ok(fn, "hipGraphInstantiate", ei);
            }
        }
    }
    if (!hip_ok(fn, "hipEventRecord", hipEventRecord(md->ev[0], md->stream)))
        return false;
    const int replays = steps - done;
    for (; done < steps; ++done)
        if (!hip_ok(fn, "hipGraphLaunch", hipGraphLaunch(g.exec, md->stream)))
            return false;
    if (!hip_ok(fn, "hipEventRecord", hipEventRecord(md->ev[1], md->stream)) ||
        !hip_ok(fn, "hipMemcpyAsync", hipMemcpyAsync(h_out, md->ring, (size_t)steps * n * 4, hipMemcpyDeviceToHost, md->stream)) ||
        !hip_ok(fn, "hipStreamSynchronize", hipStreamSynchronize(md->stream)))
        return false;
    if (h_ms)
    {
        float ms = 0.0f;
        if (replays && !hip_ok(fn, "hipEventElapsedTime", hipEventElapsedTime(&ms, md->ev[0], md->ev[1])))
            return false;
        *h_ms = replays ? ms * (float)steps / (float)replays : 0.0f;
    }
    return true;
}

extern "C" bool llam_seqm_trace(void *model, float *h_trace)
{
    Model *md = static_cast<Model *>(model);
    if (!md)
        return fail("trace", "null model");
    md->trace = h_trace;
    return true;
}

extern "C" size_t llam_seqm_slot_bytes(void *model) { return model ? static_cast<Model *>(model)->slot_bytes : 0; }
extern "C" size_t llam_seqm_device_bytes(void *model) { return model ? static_cast<Model *>(model)->owned_bytes : 0; }
