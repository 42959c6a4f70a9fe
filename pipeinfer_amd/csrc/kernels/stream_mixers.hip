// Operators of blocks whose residual is several streams mixed by small learned matrices, of a matrix memory with exponential gates and a normaliser, and of latent attention behind two latents
// with a rotated key part and a sliding window.  Everything here is fp32 in both precisions of the engine: streams, norms, gates and their running maximum, angles.
//
//   k_hyper_step       x_t <- sum_s mix[s][t] x_s + out[t] y over the streams of a token, the next sublayer's input sum_s in[s] x_s and its RMS norm in one pass over the row
//                      (one stream: the plain pre-norm residual, x <- x + y [+ a fixed vector], and the norm of what reads it next)
//   k_memory_gates     capped log gates and their running maximum (a max-plus scan over the tokens of a sequence), as factors the linear recurrence takes per token
//   k_memory_norm      the memory's output divided by its normaliser, per-head RMS norm, weight, output gate
//   k_window_mask      the pass's mask rows restricted to a window of positions
//   k_latent_prepare   both latents of a token normed, the shared key part rotated; the key / value row goes to the token's cache cell
// The recurrence itself is pi_op_linear_attention_keysum (hybrid.hip), the attention pi_op_latent_attention_rot.
#include "ops_common.h"
#include "kernel_timing.h"

#include <algorithm>
#include <cmath>

#define SM_FRESH (1 << 30)

static __device__ __forceinline__ float sm_sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }

// ---- the residual streams ----------------------------------------------------------------------------------------------------------------------------
// one workgroup per token; a thread owns NG groups of VEC neighbouring values of ALL streams, so the step may run in place and only the next input's squares are summed across threads
template <int S, int VEC, int NG>
__global__ void __launch_bounds__(1024) k_hyper_step(const float * xin, int64_t xts, int64_t xss, int ns, const float * __restrict__ y, int64_t ys, const float * __restrict__ mix, const float * __restrict__ outc,
                                                     const float * __restrict__ in_next, const float * __restrict__ shift, const float * __restrict__ w, float eps, int n, float * xo, float * __restrict__ h, int64_t hs,
                                                     const int32_t * __restrict__ abort_w) {
    if (pi_aborted(abort_w)) return;
    __shared__ float red[16];
    const int t = blockIdx.x;
    float u[NG][VEC], ss = 0.0f;
#pragma unroll
    for (int g = 0; g < NG; g++) {
        const int i = (threadIdx.x + g * blockDim.x) * VEC;
#pragma unroll
        for (int e = 0; e < VEC; e++) u[g][e] = 0.0f;
        if (i >= n) continue;
        float x[S][VEC], yv[VEC];
#pragma unroll
        for (int s = 0; s < S; s++) {
            const float * src = xin + (int64_t) t * xts + (int64_t) min(s, ns - 1) * xss + i;
            if constexpr (VEC == 4) { const float4 v = *(const float4 *) src; x[s][0] = v.x; x[s][1] = v.y; x[s][2] = v.z; x[s][3] = v.w; } else x[s][0] = src[0];
        }
#pragma unroll
        for (int e = 0; e < VEC; e++) yv[e] = 0.0f;
        if (y) {
            if constexpr (VEC == 4) { const float4 v = *(const float4 *) (y + (int64_t) t * ys + i); yv[0] = v.x; yv[1] = v.y; yv[2] = v.z; yv[3] = v.w; } else yv[0] = y[(int64_t) t * ys + i];
        }
#pragma unroll
        for (int d = 0; d < S; d++) if (d < ns) {
            float v[VEC];
#pragma unroll
            for (int e = 0; e < VEC; e++) v[e] = x[d][e];
            if (mix) {
#pragma unroll
                for (int e = 0; e < VEC; e++) v[e] = 0.0f;
#pragma unroll
                for (int s = 0; s < S; s++) if (s < ns) {
                    const float m = mix[s * ns + d];
#pragma unroll
                    for (int e = 0; e < VEC; e++) v[e] = fmaf(m, x[s][e], v[e]);
                }
            }
            if (y) {
                const float o = outc ? outc[d] : 1.0f;
#pragma unroll
                for (int e = 0; e < VEC; e++) v[e] = fmaf(o, yv[e], v[e]);
            }
            if (shift) {
#pragma unroll
                for (int e = 0; e < VEC; e++) v[e] += shift[i + e];
            }
            if (xo) {
                float * dst = xo + ((int64_t) t * ns + d) * n + i;
                if constexpr (VEC == 4) *(float4 *) dst = make_float4(v[0], v[1], v[2], v[3]); else dst[0] = v[0];
            }
            const float c = in_next ? in_next[d] : 1.0f;
#pragma unroll
            for (int e = 0; e < VEC; e++) u[g][e] = fmaf(c, v[e], u[g][e]);
        }
#pragma unroll
        for (int e = 0; e < VEC; e++) ss = fmaf(u[g][e], u[g][e], ss);
    }
    ss = pi_lanes_sum<64>(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    float tot = 0.0f;
    for (int i = 0; i < (int) (blockDim.x >> 6); i++) tot += red[i];
    const float inv = 1.0f / sqrtf(tot / (float) n + eps);
#pragma unroll
    for (int g = 0; g < NG; g++) {
        const int i = (threadIdx.x + g * blockDim.x) * VEC;
        if (i >= n) continue;
        float * dst = h + (int64_t) t * hs + i;
        if constexpr (VEC == 4) { const float4 wv = *(const float4 *) (w + i); *(float4 *) dst = make_float4(u[g][0] * inv * wv.x, u[g][1] * inv * wv.y, u[g][2] * inv * wv.z, u[g][3] * inv * wv.w); }
        else dst[0] = u[g][0] * inv * w[i];
    }
}
static int hyper_step(const float * x_in, int64_t token_stride, int64_t stream_stride, int streams, const float * y, int64_t y_stride, const float * mix_dev, const float * out_dev, const float * in_next_dev,
                      const float * shift_dev, const float * w_dev, float eps, int n, int n_tok, float * x_out, float * h_out, int64_t h_stride, void * stream) {
    if (n_tok <= 0 || n <= 0) return 0;
    if (streams < 1 || streams > PI_MAX_STREAMS || n > 16384) { pi_set_error("pi_op_hyper_step: %d streams of %d values (at most %d of 16384)", streams, n, PI_MAX_STREAMS); return -1; }
    if (!x_in || !w_dev || !h_out) { pi_set_error("pi_op_hyper_step: the streams, the norm's weight and its output are required"); return -1; }
    if (x_out == x_in && (stream_stride != n || token_stride != (int64_t) streams * n)) { pi_set_error("pi_op_hyper_step: in place the streams lie as they are stored"); return -1; }
    auto al = [](const void * p, int64_t stride) { return !p || (((uintptr_t) p % 16) == 0 && stride % 4 == 0); };
    const bool vec = n % 4 == 0 && al(x_in, token_stride) && stream_stride % 4 == 0 && al(y, y_stride) && al(w_dev, 0) && al(x_out, 0) && al(h_out, h_stride);
    const int groups = (n + (vec ? 3 : 0)) / (vec ? 4 : 1), ng = groups <= 1024 ? 1 : groups <= 4096 ? 4 : 16;
    const int threads = ng > 1 ? 1024 : (groups + 63) / 64 * 64;
    const double bytes = 4.0 * n * n_tok * ((stream_stride ? streams : 1) + (y ? 1 : 0) + (x_out ? streams : 0) + 1);
#define HS_GO(S, V, G) PI_KT_LAUNCH(PI_KT_OTHER, 0, 1, bytes, (k_hyper_step<S, V, G>), dim3((unsigned) n_tok), dim3((unsigned) threads), 0, (hipStream_t) stream, x_in, token_stride, stream_stride, streams, y, y_stride, mix_dev, \
                                    out_dev, in_next_dev, shift_dev, w_dev, eps, n, x_out, h_out, h_stride, pi_abort_word())
#define HS_S(V, G) do { if (streams == 1) HS_GO(1, V, G); else if (streams == 2) HS_GO(2, V, G); else if (streams == 3) HS_GO(3, V, G); else if (streams == 4) HS_GO(4, V, G); else if (streams <= 8) HS_GO(8, V, G); else HS_GO(16, V, G); } while (0)
    if (vec) { if (ng == 1) HS_S(4, 1); else HS_S(4, 4); }
    else { if (ng == 1) HS_S(1, 1); else if (ng == 4) HS_S(1, 4); else HS_S(1, 16); }
#undef HS_S
#undef HS_GO
    PI_CHECK_LAUNCH(); return 0;
}
extern "C" int pi_op_hyper_step(const float * x_in, int64_t token_stride, int64_t stream_stride, int streams, const float * y, int64_t y_stride, const float * mix_dev, const float * out_dev, const float * in_next_dev,
                                const float * w_dev, float eps, int n, int n_tok, float * x_out, float * h_out, int64_t h_stride, void * stream) {
    if (n_tok > 0 && n > 0 && y && !out_dev) { pi_set_error("pi_op_hyper_step: the factors of a sublayer's result are required"); return -1; }
    return hyper_step(x_in, token_stride, stream_stride, streams, y, y_stride, mix_dev, out_dev, in_next_dev, nullptr, w_dev, eps, n, n_tok, x_out, h_out, h_stride, stream);
}
// the same kernel over ONE stream: x <- x + y + shift, h = R(x) * w
extern "C" int pi_op_residual_norm(const float * x_in, const float * y, int64_t y_stride, const float * shift_dev, const float * w_dev, float eps, int n, int n_tok, float * x_out, float * h_out, int64_t h_stride, void * stream) {
    return hyper_step(x_in, n, n, 1, y, y_stride, nullptr, nullptr, nullptr, shift_dev, w_dev, eps, n, n_tok, x_out, h_out, h_stride, stream);
}

// ---- gates of the matrix memory -----------------------------------------------------------------------------------------------------------------------
// one workgroup per head walks the pass 64 tokens per wave at a time.  m' = max(f + m, i) is affine in the max-plus sense: token t is the pair (f, i), two neighbours combine to (f1 + f2, max(i1 + f2, i2)).
// A sequence's first token takes the m it starts from into its i and blocks what lies before it with f = -infinity, so the runs of a pass need no loop of their own.  Every wave scans its tokens, the waves'
// totals are chained through LDS.  The factors are formed from the very m that is handed on, whatever the scan's order rounded it to.
__global__ void __launch_bounds__(1024) k_memory_gates(const float * __restrict__ ri, const float * __restrict__ rf, int64_t stride, const float * __restrict__ bi, const float * __restrict__ bf, float cap, int heads,
                                                       float * m_state, const int32_t * __restrict__ rec, int n_tok, float * __restrict__ forget, float * __restrict__ put, float * __restrict__ flo,
                                                       const int32_t * __restrict__ abort_w) {
    if (pi_aborted(abort_w)) return;
    __shared__ float tot[16][2];
    const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6;
    const float bih = bi[h], bfh = bf[h];
    float m_base = 0.0f;                                               // m ahead of this round's tokens (a pass's first token starts a run: it does not look at it)
    for (int t0 = 0; t0 < n_tok; t0 += blockDim.x) {
        const int t = t0 + threadIdx.x;
        const bool ok = t < n_tok;
        const int word = ok ? rec[t] : -1, slot = word & ~SM_FRESH;
        const bool first = ok && (t == 0 || (rec[t - 1] & ~SM_FRESH) != slot), last = ok && (t + 1 == n_tok || (rec[t + 1] & ~SM_FRESH) != slot);
        const float i = ok ? cap * tanhf((ri[(int64_t) t * stride + h] + bih) / cap) : -INFINITY;
        const float a = ok ? cap * tanhf((rf[(int64_t) t * stride + h] + bfh) / cap) : 0.0f;
        const float f = ok ? fminf(a, 0.0f) - log1pf(expf(-fabsf(a))) : 0.0f;          // log sigmoid(a)
        const float m_in = first && !(word & SM_FRESH) ? m_state[(int64_t) slot * heads + h] : 0.0f;
        float F = first ? -INFINITY : f, M = first ? fmaxf(f + m_in, i) : i;
        for (int d = 1; d < 64; d <<= 1) {
            const float Fp = __shfl_up(F, d, 64), Mp = __shfl_up(M, d, 64);
            if (lane >= d) { M = fmaxf(Mp + F, M); F = Fp + F; }
        }
        if (t0) __syncthreads();                                       // (the previous round's totals are no longer read)
        if (lane == 63) { tot[wave][0] = F; tot[wave][1] = M; }
        __syncthreads();
        float m_wave = m_base, m_end = m_base;
        for (int w = 0; w < waves; w++) { if (w == wave) m_wave = m_end; m_end = fmaxf(m_end + tot[w][0], tot[w][1]); }
        const float m = fmaxf(m_wave + F, M);                          // behind this token
        const float prev = __shfl_up(m, 1, 64), m_prev = first ? m_in : lane == 0 ? m_wave : prev;
        if (ok) {
            const int64_t o = (int64_t) t * heads + h;
            forget[o] = expf(f + m_prev - m); put[o] = expf(i - m); flo[o] = expf(-m);
            if (last) m_state[(int64_t) slot * heads + h] = m;
        }
        m_base = m_end;
    }
}
extern "C" int pi_op_memory_gates(const float * raw_i, const float * raw_f, int64_t stride, const float * bias_i_dev, const float * bias_f_dev, float cap, int heads, float * m_state_dev, const int32_t * rec_dev, int n_tok,
                                  float * forget_dev, float * put_dev, float * floor_dev, void * stream) {
    if (n_tok <= 0) return 0;
    if (heads < 1 || !(cap > 0.0f) || !raw_i || !raw_f || !bias_i_dev || !bias_f_dev || !m_state_dev || !rec_dev) { pi_set_error("pi_op_memory_gates: raw gates, biases, a positive cap, the sequences' state and slot words are required"); return -1; }
    PI_KT_LAUNCH(PI_KT_OTHER, 0, 1, 20.0 * heads * n_tok, k_memory_gates, dim3((unsigned) heads), dim3((unsigned) std::min(1024, (n_tok + 63) / 64 * 64)), 0, (hipStream_t) stream, raw_i, raw_f, stride, bias_i_dev, bias_f_dev, cap, heads, m_state_dev, rec_dev, n_tok,
                 forget_dev, put_dev, floor_dev, pi_abort_word());
    PI_CHECK_LAUNCH(); return 0;
}

// grid (token, head): the head's row o [vdim | normaliser], divided, normed, weighted, gated
__global__ void __launch_bounds__(256) k_memory_norm(const float * __restrict__ y, int64_t ys, const float * __restrict__ flo, float q_mult, float add, int heads, int vdim, float eps, const float * __restrict__ w,
                                                     const float * __restrict__ gate, int64_t gs, int gate_act, float * __restrict__ out, int64_t os, const int32_t * __restrict__ abort_w) {
    if (pi_aborted(abort_w)) return;
    __shared__ float red[4];
    const int t = blockIdx.x, h = blockIdx.y;
    const float * r = y + (int64_t) t * ys + (int64_t) h * (vdim + 1);
    const float div = q_mult / (fmaxf(fabsf(q_mult * r[vdim]), flo[(int64_t) t * heads + h]) + add);
    float ss = 0.0f;
    for (int i = threadIdx.x; i < vdim; i += blockDim.x) { const float o = r[i] * div; ss = fmaf(o, o, ss); }
    ss = pi_lanes_sum<64>(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    float tot = 0.0f;
    for (int i = 0; i < (int) (blockDim.x >> 6); i++) tot += red[i];
    const float inv = div / sqrtf(tot / (float) vdim + eps);
    for (int i = threadIdx.x; i < vdim; i += blockDim.x) {
        float v = r[i] * inv * w[(int64_t) h * vdim + i];
        if (gate) { const float g = gate[(int64_t) t * gs + (int64_t) h * vdim + i]; v *= gate_act == PI_ACT_NONE ? g : gate_act == PI_ACT_SILU ? g * sm_sigmoid(g) : sm_sigmoid(g); }
        out[(int64_t) t * os + (int64_t) h * vdim + i] = v;
    }
}
extern "C" int pi_op_memory_norm(const float * y, int64_t y_stride, const float * floor_dev, float q_mult, float add, int heads, int vdim, float eps, const float * w_dev, const float * gate_dev, int64_t gate_stride, int gate_act,
                                 int n_tok, float * out, int64_t out_stride, void * stream) {
    if (n_tok <= 0) return 0;
    if (heads < 1 || vdim < 1 || y_stride < (int64_t) heads * (vdim + 1) || out_stride < (int64_t) heads * vdim) { pi_set_error("pi_op_memory_norm: rows of %lld / %lld floats for %d heads of %d values", (long long) y_stride, (long long) out_stride, heads, vdim); return -1; }
    if (out == y) { pi_set_error("pi_op_memory_norm: input and output rows differ in width"); return -1; }
    if (gate_dev && gate_act != PI_ACT_NONE && gate_act != PI_ACT_SIGMOID && gate_act != PI_ACT_SILU) { pi_set_error("pi_op_memory_norm: gate activation %d is unknown", gate_act); return -1; }
    PI_KT_LAUNCH(PI_KT_OTHER, 0, 1, 4.0 * n_tok * heads * (vdim * (gate_dev ? 3.0 : 2.0) + 2.0), k_memory_norm, dim3((unsigned) n_tok, (unsigned) heads), dim3((unsigned) std::min(256, (vdim + 63) / 64 * 64)), 0, (hipStream_t) stream,
                 y, y_stride, floor_dev, q_mult, add, heads, vdim, eps, w_dev, gate_dev, gate_stride, gate_act, out, out_stride, pi_abort_word());
    PI_CHECK_LAUNCH(); return 0;
}

// ---- the mask of a sliding window --------------------------------------------------------------------------------------------------------------------
// grid (token, blocks of 256 mask words' worth of cells).  Every workgroup writes the positions of ALL cells of the pass before it looks at any (the same values from everyone), so none waits for another
__global__ void __launch_bounds__(256) k_window_mask(const uint32_t * __restrict__ mask, const int32_t * __restrict__ pos, int32_t * cell_pos, int size, int n_tok, int n_kv_arg, uint32_t * __restrict__ out,
                                                     const int32_t * __restrict__ dyn, const int32_t * __restrict__ abort_w) {
    if (pi_aborted(abort_w)) return;
    for (int t = threadIdx.x; t < n_tok; t += 256) cell_pos[pi_cell_of(dyn, 0, t)] = pos[t];
    __syncthreads();
    const int t = blockIdx.x, words = (n_kv_arg + 31) / 32, n_kv = min(dyn[1], n_kv_arg);
    const int first = pos[t] - size + 1;
    const uint32_t * mrow = mask + (int64_t) t * words;
    uint32_t * orow = out + (int64_t) t * words;
    // half a wave per word: lane = cell
    const int lane = threadIdx.x & 31;
    for (int w = blockIdx.y * 256 + (threadIdx.x >> 5); w < min(words, (int) blockIdx.y * 256 + 256); w += 8) {
        const int c = w * 32 + lane;
        const uint32_t bits = w * 32 < n_kv ? mrow[w] : 0u;            // (words behind the cells in use are not written by the host)
        const bool in = c < n_kv && ((bits >> lane) & 1u) && cell_pos[c] >= first;
        const unsigned long long b = __ballot(in);
        if (lane == 0) orow[w] = (uint32_t) ((threadIdx.x & 32) ? b >> 32 : b);
    }
}
extern "C" int pi_op_window_mask(const uint32_t * mask_dev, const int32_t * pos_dev, int32_t * cell_pos_dev, int size, int n_tok, int n_kv, uint32_t * out_mask_dev, const int32_t * dyn_dev, void * stream) {
    if (n_tok <= 0 || n_kv <= 0) return 0;
    if (size < 1 || !dyn_dev || !cell_pos_dev || out_mask_dev == mask_dev) { pi_set_error("pi_op_window_mask: a window of %d positions (at least 1), the pass's cell table, the cells' positions and rows of its own are required", size); return -1; }
    const int words = (n_kv + 31) / 32;
    PI_KT_LAUNCH(PI_KT_OTHER, 0, 1, 4.0 * n_tok * (2.0 * words + n_kv), k_window_mask, dim3((unsigned) n_tok, (unsigned) ((words + 255) / 256)), dim3(256), 0, (hipStream_t) stream, mask_dev, pos_dev, cell_pos_dev, size, n_tok, n_kv,
                 out_mask_dev, dyn_dev, pi_abort_word());
    PI_CHECK_LAUNCH(); return 0;
}

// ---- the two latents -----------------------------------------------------------------------------------------------------------------------------------
// grid (token, 2): the query latent; the key / value latent and the rotated key part
__global__ void __launch_bounds__(256) k_latent_prepare(const float * __restrict__ p, int64_t ps, int q_rank, const float * __restrict__ qw, int rank, const float * __restrict__ kw, int rot, const float2 * __restrict__ cs,
                                                        int n_pos, int pairing, float eps, const int32_t * __restrict__ pos, float * __restrict__ cq, int64_t cqs, float * __restrict__ cache, const int32_t * __restrict__ dyn,
                                                        const int32_t * __restrict__ abort_w) {
    if (pi_aborted(abort_w)) return;
    __shared__ float red[4];
    const int t = blockIdx.x, tid = threadIdx.x;
    const bool is_q = blockIdx.y == 0;
    const int n = is_q ? q_rank : rank;
    const float * src = p + (int64_t) t * ps + (is_q ? 0 : q_rank), * w = is_q ? qw : kw;
    float ss = 0.0f;
    for (int i = tid; i < n; i += 256) ss = fmaf(src[i], src[i], ss);
    ss = pi_lanes_sum<64>(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float) n + eps);
    float * dst = is_q ? cq + (int64_t) t * cqs : cache + (int64_t) pi_cell_of(dyn, 0, t) * (rank + rot);
    for (int i = tid; i < n; i += 256) dst[i] = src[i] * inv * w[i];
    if (is_q) return;
    const float2 * row = cs + (int64_t) min(pos[t], n_pos - 1) * (rot / 2);
    for (int i = tid; i < rot; i += 256) {
        const pi_turn u = pi_turn_of(i, rot / 2, pairing);
        const float2 c = row[u.angle];
        const float own = src[rank + i], other = src[rank + u.mate];
        dst[rank + i] = u.lead ? own * c.x - other * c.y : own * c.x + other * c.y;
    }
}
extern "C" int pi_op_latent_prepare(const float * p, int64_t p_stride, int q_rank, const float * q_norm_w, int kv_rank, const float * kv_norm_w, int rot_dim, const void * rotary_table, float eps, const int32_t * pos_dev, int n_tok,
                                    float * q_latent, int64_t q_latent_stride, float * cache_dev, const int32_t * dyn_dev, void * stream) {
    return pi_op_latent_prepare_ex(p, p_stride, q_rank, q_norm_w, kv_rank, kv_norm_w, rot_dim, rotary_table, PI_PAIR_NEIGHBOURS, eps, pos_dev, n_tok, q_latent, q_latent_stride, cache_dev, dyn_dev, stream);
}
extern "C" int pi_op_latent_prepare_ex(const float * p, int64_t p_stride, int q_rank, const float * q_norm_w, int kv_rank, const float * kv_norm_w, int rot_dim, const void * rotary_table, int pairing, float eps, const int32_t * pos_dev,
                                       int n_tok, float * q_latent, int64_t q_latent_stride, float * cache_dev, const int32_t * dyn_dev, void * stream) {
    if (n_tok <= 0) return 0;
    const float2 * cs = nullptr; int n_pos = 0, half = 0;
    pi_rotary_table_view(rotary_table, &cs, &n_pos, &half);
    if (q_rank < 1 || kv_rank < 1 || rot_dim < 0 || (rot_dim & 1) || (rot_dim > 0 && (!cs || half != rot_dim / 2 || !pos_dev)) || (pairing != PI_PAIR_HALVES && pairing != PI_PAIR_NEIGHBOURS)) { pi_set_error("pi_op_latent_prepare: latents of %d and %d values, %d rotated ones with a table over them", q_rank, kv_rank, rot_dim); return -1; }
    if (p_stride < (int64_t) q_rank + kv_rank + rot_dim || q_latent_stride < q_rank || !dyn_dev || !q_norm_w || !kv_norm_w) { pi_set_error("pi_op_latent_prepare: row strides below the sizes, or no norm weights / cell table"); return -1; }
    PI_KT_LAUNCH(PI_KT_OTHER, 0, 1, 8.0 * n_tok * (q_rank + kv_rank + rot_dim), k_latent_prepare, dim3((unsigned) n_tok, 2), dim3(256), 0, (hipStream_t) stream, p, p_stride, q_rank, q_norm_w, kv_rank, kv_norm_w, rot_dim, cs, n_pos, pairing, eps, pos_dev,
                 q_latent, q_latent_stride, cache_dev, dyn_dev, pi_abort_word());
    PI_CHECK_LAUNCH(); return 0;
}
