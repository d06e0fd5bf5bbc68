// Gated delta rule behind short convolutions (per head a state S [dim x vdim]), for gfx950.
//
// All of the recurrence is 32-bit in both number formats: unit vectors, gates, products (on
// v_mfma_f32_16x16x4_f32 in prompts) and state; the format matters only for the output rows.
//
// Decoding: a workgroup per head and sequence does the whole step.  A thread's part of S is read once; since
//   S' q = (decay S)^T q + u (k . q),   u = beta (v - decay S^T k),
// one sum over the rows of S serves the write and the read-out.
//
// Prompts run in chunks of DC tokens.  With G_t the sum of the log decays from the chunk's start to t, the
// writes u_t of a chunk solve a unit triangular system whose right side is linear in the state S_0 before it:
//   u_t + sum_{j<t} A_tj u_j = beta_t v_t - (beta_t e^(G_t) k_t)^T S_0,   A_tj = beta_t e^(G_t - G_j) (k_t . k_j)
//   u = U - W S_0      (U, W: the system solved for the v and the k part)
//   o_t = e^(G_t) q_t^T S_0 + sum_{j<=t} P_tj u_j,   P_tj = e^(G_t - G_j) (q_t . k_j)
//   S_end = e^(G_end) S_0 + sum_j e^(G_end - G_j) k_j u_j^T
// in four launches: convolutions, unit vectors and gates of all tokens; A, P, U and W of all chunks (a thread
// solves one column by substitution, the column in its registers); the walk over the chunks, where a workgroup
// owns 16 columns of S from the first chunk to the last; head norm and output gate.  Sums of log decays are kept
// in double, because their differences enter exponentials.
#include "seq_common.h"
#include "llaminar_amd/seq_api.h"

namespace llamql
{
    constexpr int DC = 64;             // tokens of a chunk
    constexpr int DELTA_DIM_MAX = 256; // a wavefront holds a q or k vector, four values a lane

    struct DeltaArgs
    {
        llam_seq_delta_args a;
        const int32_t *row0, *ntok, *slot, *pos;
        int entry, rows, channels; // rows: tokens the scratch is laid out for
        float *q, *k, *v;          // [kv_heads][rows][dim] twice, [heads][rows][vdim]
        float *beta, *log_decay;   // [heads][rows]
        float *P, *U, *W, *kd;     // per chunk and head: [DC][DC], [DC][vdim], [DC][dim], [dim][DC]
        float *gamma;              // per chunk and head: e^(G_t), [DC], then e^(G_end)
        float *o;                  // [rows][heads][vdim]
    };

    __device__ __forceinline__ void delta_gates(const llam_seq_delta_args &p, const float *row, int h, float &beta, float &log_decay)
    {
        const float *raw = row + 2 * p.kv_heads * p.dim + 2 * p.heads * p.vdim;
        beta = sigmoidf(raw[h]);
        const float z = raw[p.heads + h] + p.d_dt_bias[h];
        log_decay = -expf(p.d_a_log[h]) * (fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))));
    }

    // Convolution and silu of channels ch .. ch + 3 for the token at row `r` and position `pos` of an entry that
    // starts at pos0: earlier inputs of this step from the projection, others from the sequence's recent ones.
    __device__ __forceinline__ f32x4 delta_conv(const DeltaArgs &p, int r, int pos, int pos0, int slot, int ch)
    {
        f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
        const int taps = p.a.taps;
        const float *recent = p.a.d_recent + (size_t)slot * taps * p.channels;
        const int place = pos % taps;
        for (int b0 = 0; b0 < taps; b0 += 4) // (four taps at a time, their inputs all requested before the first is used)
        {
            f32x4 x[4], w[4];
#pragma unroll
            for (int i = 0; i < 4; ++i)
            {
                const int back = b0 + i < taps ? b0 + i : taps - 1, at = pos - back;
                const float *row = at >= pos0 ? p.a.d_proj + (size_t)(r - back) * p.a.ldp
                                              : recent + (size_t)(back <= place ? place - back : place - back + taps) * p.channels;
                x[i] = *reinterpret_cast<const f32x4 *>(row + ch);
                w[i] = *reinterpret_cast<const f32x4 *>(p.a.d_conv + (size_t)(taps - 1 - back) * p.channels + ch);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int k = 0; k < 4; ++k) // before the sequence's start there is nothing, whatever the state holds
                    y[k] += b0 + i < taps && pos >= b0 + i ? w[i][k] * x[i][k] : 0.0f;
        }
#pragma unroll
        for (int i = 0; i < 4; ++i)
            y[i] *= sigmoidf(y[i]);
        return y;
    }

    // the factor that makes a vector a unit vector, four of its values in each of `lanes` neighbouring lanes
    __device__ __forceinline__ float delta_unit(f32x4 y, int lanes)
    {
        float sum = y[0] * y[0] + y[1] * y[1] + y[2] * y[2] + y[3] * y[3];
        for (int off = lanes / 2; off > 0; off >>= 1)
            sum += __shfl_xor(sum, off, 64);
        return 1.0f / sqrtf(sum + 1e-6f);
    }

    // ---- decoding -------------------------------------------------------------------------------
    // NR: rows of S a thread holds (dim = 16 NR); 128 columns at a time.
    constexpr int STEP_THREADS = 512;
    template <typename T, int NR>
    __global__ void __launch_bounds__(STEP_THREADS)
        delta_step_kernel(DeltaArgs p)
    {
        typedef T t4 __attribute__((ext_vector_type(4)));
        extern __shared__ __attribute__((aligned(16))) float s_v[]; // [vdim], then the outputs [vdim]
        __shared__ __attribute__((aligned(16))) float s_q[DELTA_DIM_MAX], s_k[DELTA_DIM_MAX], s_part[STEP_THREADS / 64][2][128];
        __shared__ float s_sum[STEP_THREADS / 64];
        const llam_seq_delta_args &a = p.a;
        const int h = blockIdx.x, e = p.entry + blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
        const int r = p.row0[e], slot = p.slot[e], pos = p.pos[e];
        const int per = a.heads / a.kv_heads, kv = h / per, dim = 16 * NR;
        const bool fresh = pos == 0;
        const float *row = a.d_proj + (size_t)r * a.ldp;
        float *S = a.d_state + ((size_t)slot * a.heads + h) * dim * a.vdim;
        float *s_o = s_v + a.vdim;
        const int d0 = threadIdx.x >> 5, cc = (threadIdx.x & 31) * 4;

        f32x4 s[NR];
        auto fetch = [&](int col) __attribute__((always_inline)) {
#pragma unroll
            for (int i = 0; i < NR; ++i)
            {
                s[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
                if (!fresh && col < a.vdim)
                    s[i] = *reinterpret_cast<const f32x4 *>(S + (size_t)(d0 + 16 * i) * a.vdim + col);
            }
        };
        fetch(cc); // requested before the convolutions are worked out
        float *keep = a.d_recent + ((size_t)slot * a.taps + pos % a.taps) * p.channels;
        if (wave < 2)
        {
            // q, k
            const int ch = (wave * a.kv_heads + kv) * dim + lane * 4;
            f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
            if (lane * 4 < dim)
                y = delta_conv(p, r, pos, pos, slot, ch);
            y = y * (delta_unit(y, 64) * (wave == 0 ? 1.0f / sqrtf((float)a.dim_real) : 1.0f));
            if (lane * 4 < dim)
            {
                *reinterpret_cast<f32x4 *>((wave == 0 ? s_q : s_k) + lane * 4) = y;
                if (h == kv * per)
                    *reinterpret_cast<f32x4 *>(keep + ch) = *reinterpret_cast<const f32x4 *>(row + ch);
            }
        }
        else
            for (int d = (threadIdx.x - 128) * 4; d < a.vdim; d += (STEP_THREADS - 128) * 4)
            {
                const int ch = 2 * a.kv_heads * dim + h * a.vdim + d;
                *reinterpret_cast<f32x4 *>(s_v + d) = delta_conv(p, r, pos, pos, slot, ch);
                *reinterpret_cast<f32x4 *>(keep + ch) = *reinterpret_cast<const f32x4 *>(row + ch);
            }
        float beta, log_decay;
        delta_gates(a, row, h, beta, log_decay);
        const float decay = expf(log_decay);
        __syncthreads();
        float kq = 0.0f;
#pragma unroll
        for (int i = 0; i < (NR + 3) / 4; ++i)
            if (lane + 64 * i < dim)
                kq += s_q[lane + 64 * i] * s_k[lane + 64 * i];
        kq = wave_sum64(kq);

        float sum = 0.0f;
        for (int c0 = 0; c0 < a.vdim; c0 += 128)
        {
            if (c0)
            {
                fetch(c0 + cc);
                __syncthreads();
            }
            f32x4 rk = {0.0f, 0.0f, 0.0f, 0.0f}, rq = rk;
#pragma unroll
            for (int i = 0; i < NR; ++i)
            {
                rk = rk + s[i] * s_k[d0 + 16 * i];
                rq = rq + s[i] * s_q[d0 + 16 * i];
            }
#pragma unroll
            for (int j = 0; j < 4; ++j)
            {
                rk[j] += __shfl_xor(rk[j], 32, 64);
                rq[j] += __shfl_xor(rq[j], 32, 64);
            }
            if (lane < 32)
            {
                *reinterpret_cast<f32x4 *>(&s_part[wave][0][cc]) = rk;
                *reinterpret_cast<f32x4 *>(&s_part[wave][1][cc]) = rq;
            }
            __syncthreads();
            if (c0 + cc < a.vdim)
            {
                rk = rq = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                for (int w = 0; w < STEP_THREADS / 64; ++w)
                {
                    rk = rk + *reinterpret_cast<const f32x4 *>(&s_part[w][0][cc]);
                    rq = rq + *reinterpret_cast<const f32x4 *>(&s_part[w][1][cc]);
                }
                const f32x4 u = (*reinterpret_cast<const f32x4 *>(s_v + c0 + cc) - rk * decay) * beta;
                if (d0 == 0)
                {
                    const f32x4 o = rq * decay + u * kq;
                    *reinterpret_cast<f32x4 *>(s_o + c0 + cc) = o;
                    sum += o[0] * o[0] + o[1] * o[1] + o[2] * o[2] + o[3] * o[3];
                }
#pragma unroll
                for (int i = 0; i < NR; ++i)
                    *reinterpret_cast<f32x4 *>(S + (size_t)(d0 + 16 * i) * a.vdim + c0 + cc) = s[i] * decay + u * s_k[d0 + 16 * i];
            }
        }
        sum = block_sum<STEP_THREADS>(sum, s_sum); // (its barriers publish s_o)
        const float scale = 1.0f / sqrtf(sum / (float)a.vdim_real + a.eps);
        const float *gate = row + 2 * a.kv_heads * dim + (a.heads + h) * a.vdim;
        T *y = static_cast<T *>(a.d_y) + (size_t)r * a.ldy + h * a.vdim;
        for (int d = threadIdx.x * 4; d < a.vdim; d += STEP_THREADS * 4)
        {
            f32x4 o = *reinterpret_cast<const f32x4 *>(s_o + d) * scale * *reinterpret_cast<const f32x4 *>(a.d_norm + d);
            const f32x4 z = *reinterpret_cast<const f32x4 *>(gate + d);
#pragma unroll
            for (int j = 0; j < 4; ++j)
                o[j] *= z[j] * sigmoidf(z[j]);
            *reinterpret_cast<t4 *>(y + d) = __builtin_convertvector(o, t4);
        }
    }

    // ---- prompts: convolutions, unit vectors, gates -------------------------------------------------
    // Workgroup = INPUT_TOKENS neighbouring tokens of one vector (q heads, k heads, v heads), 16, 32 or 64 lanes
    // per token: a token's inputs are used by the next ones' taps while they are near.
    constexpr int INPUT_TOKENS = 16;
    __global__ void __launch_bounds__(256)
        delta_inputs_kernel(DeltaArgs p)
    {
        const llam_seq_delta_args &a = p.a;
        const int e = p.entry, n = p.ntok[e], unit = blockIdx.x, G = a.kv_heads;
        const int slot = p.slot[e], pos0 = p.pos[e];
        const int size = unit < 2 * G ? a.dim : a.vdim, lanes = size <= 64 ? 16 : size <= 128 ? 32 : 64;
        const int lane = threadIdx.x & (lanes - 1);
        for (int i = threadIdx.x / lanes; i < INPUT_TOKENS; i += 256 / lanes)
        {
            const int t = blockIdx.y * INPUT_TOKENS + i, r = p.row0[e] + t;
            if (t >= n) // (lanes of one vector leave together)
                return;
            if (unit < 2 * G)
            {
                const bool query = unit < G;
                f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
                if (lane * 4 < a.dim)
                    y = delta_conv(p, r, pos0 + t, pos0, slot, unit * a.dim + lane * 4);
                y = y * (delta_unit(y, lanes) * (query ? 1.0f / sqrtf((float)a.dim_real) : 1.0f));
                if (lane * 4 < a.dim)
                    *reinterpret_cast<f32x4 *>((query ? p.q : p.k) + ((size_t)(query ? unit : unit - G) * p.rows + t) * a.dim + lane * 4) = y;
            }
            else
            {
                const int h = unit - 2 * G;
                for (int d = lane * 4; d < a.vdim; d += lanes * 4)
                    *reinterpret_cast<f32x4 *>(p.v + ((size_t)h * p.rows + t) * a.vdim + d) = delta_conv(p, r, pos0 + t, pos0, slot, 2 * G * a.dim + h * a.vdim + d);
                if (lane == 0)
                    delta_gates(a, a.d_proj + (size_t)r * a.ldp, h, p.beta[(size_t)h * p.rows + t], p.log_decay[(size_t)h * p.rows + t]);
            }
        }
    }

    // The portion's last inputs become the sequence's recent ones (after the convolutions have read the old ones).
    __global__ void __launch_bounds__(256)
        delta_keep_kernel(DeltaArgs p)
    {
        const int e = p.entry, n = p.ntok[e], back = blockIdx.y; // back = 0: the last token
        const int ch = (blockIdx.x * 256 + threadIdx.x) * 4;
        if (back >= n || ch >= p.channels)
            return;
        const int at = p.pos[e] + n - 1 - back;
        *reinterpret_cast<f32x4 *>(p.a.d_recent + ((size_t)p.slot[e] * p.a.taps + at % p.a.taps) * p.channels + ch) =
            *reinterpret_cast<const f32x4 *>(p.a.d_proj + (size_t)(p.row0[e] + n - 1 - back) * p.a.ldp + ch);
    }

    // ---- prompts: within the chunks -------------------------------------------------------------------
    __global__ void __launch_bounds__(256)
        delta_chunk_kernel(DeltaArgs p)
    {
        using O = Operand<float>;
        constexpr int LD = DC + 4;
        __shared__ __attribute__((aligned(16))) float s_A[DC][LD];
        __shared__ double s_G[DC];
        __shared__ float s_beta[DC], s_in[DC], s_out[DC]; // beta_t e^(G_t), e^(G_end - G_t)
        const llam_seq_delta_args &a = p.a;
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane & 15, g = lane >> 4;
        const int h = blockIdx.y, chunk = blockIdx.x, t0 = chunk * DC, dim = a.dim;
        const int n = p.ntok[p.entry] - t0 < DC ? p.ntok[p.entry] - t0 : DC;
        if (n <= 0)
            return;
        const int kv = h / (a.heads / a.kv_heads);
        const float *q = p.q + ((size_t)kv * p.rows + t0) * dim, *k = p.k + ((size_t)kv * p.rows + t0) * dim;
        const float *v = p.v + ((size_t)h * p.rows + t0) * a.vdim;
        const size_t job = (size_t)chunk * a.heads + h;
        auto clamp = [&](int t) { return t < n ? t : n - 1; };
        if (wave == 0)
        {
            const bool in = lane < n;
            double G = in ? (double)p.log_decay[(size_t)h * p.rows + t0 + lane] : 0.0;
#pragma unroll
            for (int off = 1; off < 64; off <<= 1)
            {
                const double o = __shfl_up(G, off, 64);
                if (lane >= off)
                    G += o;
            }
            const double end = __shfl(G, 63, 64);
            const float beta = in ? p.beta[(size_t)h * p.rows + t0 + lane] : 0.0f, carried = expf((float)G);
            s_G[lane] = G;
            s_beta[lane] = beta;
            s_in[lane] = beta * carried;
            s_out[lane] = in ? expf((float)(end - G)) : 0.0f;
            float *gamma = p.gamma + job * (DC + 4);
            gamma[lane] = carried;
            if (lane == 0)
                gamma[DC] = expf((float)end);
        }
        __syncthreads();

        // rows 16 wave .. of k k^T and q k^T, up to the diagonal
        {
            f32x4 kk[DC / 16], qk[DC / 16];
#pragma unroll
            for (int j = 0; j < DC / 16; ++j)
                kk[j] = qk[j] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            const size_t mine = (size_t)clamp(wave * 16 + c) * dim + 8 * g;
            for (int s = 0; s < dim; s += 32)
            {
                const f32x8 ka = O::load(k + mine + s), qa = O::load(q + mine + s);
#pragma unroll
                for (int j = 0; j < DC / 16; ++j)
                    if (j <= wave)
                    {
                        const f32x8 b = O::load(k + (size_t)clamp(j * 16 + c) * dim + 8 * g + s);
                        kk[j] = O::mma(ka, b, kk[j]);
                        qk[j] = O::mma(qa, b, qk[j]);
                    }
            }
            float *P = p.P + job * DC * DC;
#pragma unroll
            for (int j = 0; j < DC / 16; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r)
                {
                    const int t = wave * 16 + 4 * g + r, tj = j * 16 + c;
                    const float f = tj <= t && t < n ? expf((float)(s_G[t] - s_G[tj])) : 0.0f;
                    P[t * DC + tj] = f * qk[j][r];
                    s_A[t][tj] = tj < t ? s_beta[t] * f * kk[j][r] : 0.0f;
                }
        }
        __syncthreads();

        // a thread solves one column: of k (for W), then of v (for U)
        for (int col = threadIdx.x; col < dim + a.vdim; col += 256)
        {
            const bool key = col < dim;
            const float *src = key ? k + col : v + col - dim, *gate = key ? s_in : s_beta;
            const int ld = key ? dim : a.vdim;
            float x[DC];
#pragma unroll
            for (int t = 0; t < DC; ++t)
                x[t] = src[(size_t)clamp(t) * ld];
            if (key)
            {
                float *kd = p.kd + (job * dim + col) * DC;
#pragma unroll
                for (int t = 0; t < DC; t += 4)
                    *reinterpret_cast<f32x4 *>(kd + t) = f32x4{x[t], x[t + 1], x[t + 2], x[t + 3]} * *reinterpret_cast<const f32x4 *>(s_out + t);
            }
#pragma unroll
            for (int t = 0; t < DC; ++t)
                x[t] *= gate[t];
#pragma unroll
            for (int t = 1; t < DC; ++t)
            {
                f32x4 y = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                for (int j = 0; j < t; j += 4)
                {
                    const f32x4 A = *reinterpret_cast<const f32x4 *>(&s_A[t][j]);
#pragma unroll
                    for (int i = 0; i < 4; ++i)
                        if (j + i < t)
                            y[i] += A[i] * x[j + i];
                }
                x[t] -= (y[0] + y[1]) + (y[2] + y[3]);
                __builtin_amdgcn_sched_barrier(0); // (rows of A are not all requested at once)
            }
            float *dst = key ? p.W + job * DC * dim + col : p.U + job * DC * a.vdim + col - dim;
#pragma unroll
            for (int t = 0; t < DC; ++t)
                dst[(size_t)t * ld] = x[t];
        }
    }

    // ---- prompts: the walk over the chunks --------------------------------------------------------------
    // Workgroup = 16 columns of one head's S; wavefront w computes tokens 16 w .. of a chunk and holds rows
    // w DP / 4 .. of S in its accumulators.  S and u pass between the wavefronts through LDS, column by column.
    template <int DP>
    __global__ void __launch_bounds__(256)
        delta_walk_kernel(DeltaArgs p)
    {
        using O = Operand<float>;
        constexpr int KS = DP / 32, TS = DP / 64;
        __shared__ __attribute__((aligned(16))) float s_S[16][DP + 4], s_u[16][DC + 4];
        const llam_seq_delta_args &a = p.a;
        const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, c = lane & 15, g = lane >> 4;
        // the columns of a head read the same rows: they go to one die (blocks are dealt round robin over eight)
        const int blocks = a.vdim / 16, h = blockIdx.x / (8 * blocks) * 8 + (blockIdx.x & 7);
        if (h >= a.heads)
            return;
        const int e = p.entry, ntok = p.ntok[e];
        const int kv = h / (a.heads / a.kv_heads), col = (blockIdx.x >> 3) % blocks * 16 + c;
        const bool fresh = p.pos[e] == 0;
        float *state = a.d_state + ((size_t)p.slot[e] * a.heads + h) * DP * a.vdim + col;
        const float *qrows = p.q + (size_t)kv * p.rows * DP;

        f32x4 S[TS];
#pragma unroll
        for (int i = 0; i < TS; ++i)
        {
            const int d = (wave * TS + i) * 16 + 4 * g;
            S[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            if (!fresh)
            {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    S[i][r] = state[(size_t)(d + r) * a.vdim];
            }
            *reinterpret_cast<f32x4 *>(&s_S[c][d]) = S[i];
        }
        f32x8 w[KS], q[KS];
        float u0[4];
        auto request = [&](int t0) __attribute__((always_inline)) {
            const size_t job = (size_t)(t0 / DC) * a.heads + h;
            const float *wr = p.W + (job * DC + wave * 16 + c) * DP + 8 * g;
            const int t = t0 + wave * 16 + c;
            const float *qr = qrows + (size_t)(t < ntok ? t : ntok - 1) * DP + 8 * g;
#pragma unroll
            for (int s = 0; s < KS; ++s)
            {
                w[s] = O::load(wr + 32 * s);
                q[s] = O::load(qr + 32 * s);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r)
                u0[r] = p.U[(job * DC + wave * 16 + 4 * g + r) * a.vdim + col];
        };
        request(0);
        __syncthreads();
        for (int t0 = 0; t0 < ntok; t0 += DC)
        {
            const size_t job = (size_t)(t0 / DC) * a.heads + h;
            f32x8 P[DC / 32], kd[TS][DC / 32];
            const float *gamma = p.gamma + job * (DC + 4);
            const f32x4 carried = *reinterpret_cast<const f32x4 *>(gamma + wave * 16 + 4 * g);
            const float decay = gamma[DC];
#pragma unroll
            for (int s = 0; s < DC / 32; ++s)
            {
                P[s] = O::load(p.P + (job * DC + wave * 16 + c) * DC + 32 * s + 8 * g);
#pragma unroll
                for (int i = 0; i < TS; ++i)
                    kd[i][s] = O::load(p.kd + (job * DP + (wave * TS + i) * 16 + c) * DC + 32 * s + 8 * g);
            }
            // what the state before the chunk contributes
            f32x4 ws[2], qs[2];
            ws[0] = ws[1] = qs[0] = qs[1] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int s = 0; s < KS; ++s)
            {
                const f32x8 b = O::load(&s_S[c][32 * s + 8 * g]);
                ws[s & 1] = O::mma(w[s], b, ws[s & 1]);
                qs[s & 1] = O::mma(q[s], b, qs[s & 1]);
            }
            f32x4 u, out = (qs[0] + qs[1]) * carried;
#pragma unroll
            for (int r = 0; r < 4; ++r)
                u[r] = u0[r] - (ws[0][r] + ws[1][r]);
            *reinterpret_cast<f32x4 *>(&s_u[c][wave * 16 + 4 * g]) = u;
            if (t0 + DC < ntok)
                request(t0 + DC);
            __syncthreads();
            // the chunk's own tokens, and S after it
#pragma unroll
            for (int i = 0; i < TS; ++i)
                S[i] = S[i] * decay;
#pragma unroll
            for (int s = 0; s < DC / 32; ++s)
            {
                const f32x8 b = O::load(&s_u[c][32 * s + 8 * g]);
#pragma unroll
                for (int i = 0; i < TS; ++i)
                    S[i] = O::mma(kd[i][s], b, S[i]);
                if (32 * s <= 16 * wave + 15)
                    out = O::mma(P[s], b, out);
            }
#pragma unroll
            for (int i = 0; i < TS; ++i)
                *reinterpret_cast<f32x4 *>(&s_S[c][(wave * TS + i) * 16 + 4 * g]) = S[i];
#pragma unroll
            for (int r = 0; r < 4; ++r)
            {
                const int t = t0 + wave * 16 + 4 * g + r;
                if (t < ntok)
                    p.o[((size_t)t * a.heads + h) * a.vdim + col] = out[r];
            }
            __syncthreads();
        }
#pragma unroll
        for (int i = 0; i < TS; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r)
                state[(size_t)((wave * TS + i) * 16 + 4 * g + r) * a.vdim] = S[i][r];
    }

    // ---- prompts: head norm, output gate: a wavefront per token and head ----------------------------------
    template <typename T>
    __global__ void __launch_bounds__(256)
        delta_output_kernel(DeltaArgs p)
    {
        typedef T t4 __attribute__((ext_vector_type(4)));
        const llam_seq_delta_args &a = p.a;
        const int lane = threadIdx.x & 63, h = blockIdx.x * 4 + (threadIdx.x >> 6), t = blockIdx.y;
        if (h >= a.heads)
            return;
        const int r = p.row0[p.entry] + t;
        const float *o = p.o + ((size_t)t * a.heads + h) * a.vdim;
        const float *gate = a.d_proj + (size_t)r * a.ldp + 2 * a.kv_heads * a.dim + (a.heads + h) * a.vdim;
        float sum = 0.0f;
        for (int d = lane * 4; d < a.vdim; d += 256)
        {
            const f32x4 x = *reinterpret_cast<const f32x4 *>(o + d);
            sum += x[0] * x[0] + x[1] * x[1] + x[2] * x[2] + x[3] * x[3];
        }
        const float scale = 1.0f / sqrtf(wave_sum64(sum) / (float)a.vdim_real + a.eps);
        T *y = static_cast<T *>(a.d_y) + (size_t)r * a.ldy + h * a.vdim;
        for (int d = lane * 4; d < a.vdim; d += 256)
        {
            f32x4 x = *reinterpret_cast<const f32x4 *>(o + d) * scale * *reinterpret_cast<const f32x4 *>(a.d_norm + d);
            const f32x4 z = *reinterpret_cast<const f32x4 *>(gate + d);
#pragma unroll
            for (int j = 0; j < 4; ++j)
                x[j] *= z[j] * sigmoidf(z[j]);
            *reinterpret_cast<t4 *>(y + d) = __builtin_convertvector(x, t4);
        }
    }

    namespace
    {
        struct DeltaScratch
        {
            size_t q, k, v, beta, log_decay, P, U, W, kd, gamma, o, total;
        };
        DeltaScratch delta_scratch(int rows, int heads, int kv_heads, int dim, int vdim)
        {
            DeltaScratch s{};
            size_t at = 0;
            auto take = [&at](size_t floats) {
                const size_t here = at;
                at += (floats * 4 + 255) & ~(size_t)255;
                return here;
            };
            const size_t jobs = (size_t)ceil_div(rows, DC) * heads;
            s.q = take((size_t)kv_heads * rows * dim), s.k = take((size_t)kv_heads * rows * dim), s.v = take((size_t)heads * rows * vdim);
            s.beta = take((size_t)heads * rows), s.log_decay = take((size_t)heads * rows);
            s.P = take(jobs * DC * DC), s.U = take(jobs * DC * vdim), s.W = take(jobs * DC * dim), s.kd = take(jobs * dim * DC);
            s.gamma = take(jobs * (DC + 4)), s.o = take((size_t)rows * heads * vdim);
            s.total = at;
            return s;
        }

        bool delta_args(const char *fn, const llam_seq_delta_args *a, const llam_seq_entries *e, int dtype, DeltaArgs &p)
        {
            if (!a || !e || !a->d_proj || !a->d_conv || !a->d_a_log || !a->d_dt_bias || !a->d_norm || !a->d_state || !a->d_recent || !a->d_y ||
                !e->d_row0 || !e->d_ntok || !e->d_slot || !e->d_pos)
                return fail(fn, "null pointer");
            if (dtype != LLAM_SEQ_BF16 && dtype != LLAM_SEQ_F32)
                return fail(fn, "dtype %d", dtype);
            if (a->heads < 1 || a->heads > 65535 || a->kv_heads < 1 || (a->heads % a->kv_heads) != 0)
                return fail(fn, "heads=%d must be a multiple of kv_heads=%d", a->heads, a->kv_heads);
            if (a->dim < 1 || a->dim > DELTA_DIM_MAX || (a->dim % PAD) != 0 || a->vdim < 1 || a->vdim > 4096 || (a->vdim % PAD) != 0 ||
                a->dim_real < 1 || a->dim_real > a->dim || a->vdim_real < 1 || a->vdim_real > a->vdim)
                return fail(fn, "dim=%d vdim=%d: dim up to %d, vdim up to 4096, both multiples of %d", a->dim, a->vdim, DELTA_DIM_MAX, PAD);
            if (a->taps < 1 || a->taps > 65535)
                return fail(fn, "taps=%d", a->taps);
            if (a->ldp < 2 * a->kv_heads * a->dim + 2 * a->heads * a->vdim + 2 * a->heads || (a->ldp % 4) != 0 || !aligned16(a->d_proj) ||
                !aligned16(a->d_conv) || !aligned16(a->d_norm) || !aligned16(a->d_state) || !aligned16(a->d_recent))
                return fail(fn, "ldp=%d too small or rows misaligned", a->ldp);
            if (a->ldy < a->heads * a->vdim || (a->ldy % 8) != 0 || !aligned16(a->d_y))
                return fail(fn, "ldy=%d too small or rows misaligned", a->ldy);
            p = DeltaArgs{};
            p.a = *a;
            p.channels = 2 * a->kv_heads * a->dim + a->heads * a->vdim;
            p.row0 = e->d_row0, p.ntok = e->d_ntok, p.slot = e->d_slot, p.pos = e->d_pos;
            return true;
        }

        template <typename T, int NR>
        bool step_launch(const char *fn, const DeltaArgs &p, int n, hipStream_t st)
        {
            hipLaunchKernelGGL((delta_step_kernel<T, NR>), dim3(p.a.heads, n), dim3(STEP_THREADS), (size_t)2 * p.a.vdim * 4, st, p);
            return launched(fn);
        }
        template <typename T>
        bool step_dispatch(const char *fn, const DeltaArgs &p, int n, hipStream_t st)
        {
            return p.a.dim == 64 ? step_launch<T, 4>(fn, p, n, st) : p.a.dim == 128 ? step_launch<T, 8>(fn, p, n, st)
                   : p.a.dim == 192 ? step_launch<T, 12>(fn, p, n, st) : step_launch<T, 16>(fn, p, n, st);
        }
        template <int DP>
        bool walk_launch(const char *fn, const DeltaArgs &p, hipStream_t st)
        {
            hipLaunchKernelGGL(delta_walk_kernel<DP>, dim3(round_up(p.a.heads, 8) * (p.a.vdim / 16)), dim3(256), 0, st, p);
            return launched(fn);
        }
    } // namespace
} // namespace llamql

using namespace llamql;

extern "C" size_t llam_seq_delta_scratch_bytes(int max_rows, int heads, int kv_heads, int dim, int vdim)
{
    if (max_rows < 1 || heads < 1 || kv_heads < 1 || dim < 1 || vdim < 1)
        return 0;
    return delta_scratch(max_rows, heads, kv_heads, dim, vdim).total;
}

extern "C" bool llam_seq_delta_decode(const llam_seq_delta_args *a, const llam_seq_entries *e, int first, int n, int dtype,
                                      int device_id, void *stream)
{
    static const char *fn = "llam_seq_delta_decode";
    DeltaArgs p;
    if (n < 0 || first < 0 || n > 65535)
        return fail(fn, "bad size (first=%d n=%d)", first, n);
    if (n == 0)
        return true;
    if (!delta_args(fn, a, e, dtype, p))
        return false;
    p.entry = first;
    if (!set_device(fn, device_id))
        return false;
    return dtype == LLAM_SEQ_F32 ? step_dispatch<float>(fn, p, n, as_stream(stream)) : step_dispatch<bf16>(fn, p, n, as_stream(stream));
}

extern "C" bool llam_seq_delta_prefill(const llam_seq_delta_args *a, const llam_seq_entries *e, int entry, int ntok, void *d_scratch,
                                       size_t scratch_bytes, int dtype, int device_id, void *stream)
{
    static const char *fn = "llam_seq_delta_prefill";
    DeltaArgs p;
    if (ntok < 0 || entry < 0 || ntok > 65535)
        return fail(fn, "bad size (entry=%d ntok=%d)", entry, ntok);
    if (ntok == 0)
        return true;
    if (!delta_args(fn, a, e, dtype, p))
        return false;
    const DeltaScratch at = delta_scratch(ntok, a->heads, a->kv_heads, a->dim, a->vdim);
    if (!d_scratch || at.total > scratch_bytes)
        return fail(fn, "scratch too small");
    p.entry = entry, p.rows = ntok;
    char *s = static_cast<char *>(d_scratch);
    auto place = [s](size_t offset) { return reinterpret_cast<float *>(s + offset); };
    p.q = place(at.q), p.k = place(at.k), p.v = place(at.v), p.beta = place(at.beta), p.log_decay = place(at.log_decay);
    p.P = place(at.P), p.U = place(at.U), p.W = place(at.W), p.kd = place(at.kd), p.gamma = place(at.gamma), p.o = place(at.o);
    if (!set_device(fn, device_id))
        return false;
    hipStream_t st = as_stream(stream);
    hipLaunchKernelGGL(delta_inputs_kernel, dim3(2 * a->kv_heads + a->heads, ceil_div(ntok, INPUT_TOKENS)), dim3(256), 0, st, p);
    if (!launched(fn))
        return false;
    if (a->taps > 1)
    {
        hipLaunchKernelGGL(delta_keep_kernel, dim3(ceil_div(p.channels, 1024), a->taps - 1), dim3(256), 0, st, p);
        if (!launched(fn))
            return false;
    }
    hipLaunchKernelGGL(delta_chunk_kernel, dim3(ceil_div(ntok, DC), a->heads), dim3(256), 0, st, p);
    if (!launched(fn))
        return false;
    const bool ok = a->dim == 64 ? walk_launch<64>(fn, p, st) : a->dim == 128 ? walk_launch<128>(fn, p, st)
                    : a->dim == 192 ? walk_launch<192>(fn, p, st) : walk_launch<256>(fn, p, st);
    if (!ok)
        return false;
    const dim3 grid(ceil_div(a->heads, 4), ntok);
    if (dtype == LLAM_SEQ_F32)
        hipLaunchKernelGGL(delta_output_kernel<float>, grid, dim3(256), 0, st, p);
    else
        hipLaunchKernelGGL(delta_output_kernel<bf16>, grid, dim3(256), 0, st, p);
    return launched(fn);
}
