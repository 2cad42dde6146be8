// The state-space recurrence of the layer-list models (PS_MIX_SSD), and the matrix memory (PS_MIX_MLSTM), for a portion of tokens, in CHUNKS on the fp32 matrix cores.  Per head, with dt_t = softplus(dtraw + dt_bias),
// a_t = -exp(a_log) dt_t and c_t the running sum of a over a chunk of 64 tokens, the token-by-token scan (k_seqmix.hip) is the same as
//   U     = sum_s exp(c_end - c_s) dt_s x_s B_s^T               what a chunk adds to the state                  ssd_state_kernel, all chunks at once
//   S_in  <- exp(c_end) S_in + U                                the state in front of every chunk               ssd_pass_kernel, an element per lane, chunk after chunk
//   y_t   = exp(c_t) S_in C_t + sum_(s <= t) exp(c_t - c_s) dt_s (C_t . B_s) x_s + skip x_t                     ssd_out_kernel, all chunks at once
// Everything is fp32 (v_mfma_f32_16x16x4_f32); the running sums are kept in double, so that a difference of two of them is as good as its own size asks for.  Exponents are
// never positive.  x [T][H P], B and C [T][G N] share a row stride; the state is [H][P][N].
//
// The matrix memory with exponential gates (PS_MIX_MLSTM) is the same recurrence with q, k, v for C, B, x, a log decay f_t and a log input weight i_t of its own, everything relative
// to a running maximum m_t = max(f_t + m_(t-1), i_t), and one value column more that is 1 for every token (n; the state is [H][P + 1][N]).  With c_t the running sum of f over a
// chunk and m_in the maximum in front of it,  m_t = max(c_t + m_in, c_t + max_(s <= t) (i_s - c_s)):  mlstm_gates_kernel makes all of them at once, and from them, per token,
//   u_s = i_s - c_s,  w_t = c_t - m_t      a product inside the chunk carries exp(w_t + u_s)
//   lead_t = exp(w_t + m_in)               ... with the state in front of the chunk
//   tail_s = exp(c_end - m_end + u_s)      what token s adds to the state behind the chunk;  dec = exp(c_end + m_in - m_end) is what the state itself keeps
// (LSTM = true below; the other kernels then read these instead of making decays of their own).  A maximum is rounded to fp32 BEFORE it is used, so that the one a later step
// finds in the state is the one its numbers are relative to.
#include "ps_seq.h"

#include <algorithm>
#include <cmath>

typedef float sd_f4 __attribute__((ext_vector_type(4)));
typedef float sd_f2 __attribute__((ext_vector_type(2)));
#define SD_Q 64

static __device__ __forceinline__ float sd_softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// dt and the running sums of the chunk that starts at token t0 (tokens beyond T: dt = 0); the first wave works, every thread waits
static __device__ __forceinline__ void sd_decays(const float *dtraw, long long ldb, const float *a_log, const float *dt_bias, int h, int t0, int T, double *cs, float *dts) {
    if (threadIdx.x < SD_Q) {
        const int lane = threadIdx.x, t = t0 + lane;
        const float dt = t < T ? sd_softplus(dtraw[(long long)t * ldb + h] + dt_bias[h]) : 0.f;
        double v = (double)(-expf(a_log[h]) * dt);
#pragma unroll
        for (int o = 1; o < SD_Q; o <<= 1) {
            const double u = __shfl_up(v, o, 64);
            if (lane >= o) v += u;
        }
        cs[lane] = v;
        dts[lane] = dt;
    }
    __syncthreads();
}

// what mlstm_gates_kernel leaves: per token and head ([H][chunks * SD_Q], tokens beyond T neutral), and per chunk and head dec [chunks][H]
struct sd_gates {
    double *u, *w;
    float *lead, *tail, *dec;
};
static __device__ __forceinline__ float sd_capped(float z, float cap) { return cap > 0.f ? cap * tanhf(z / cap) : z; }
static __device__ __forceinline__ float sd_log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
// block = a head, a wave per chunk (more chunks than waves: in turns).  dynamic LDS: 2 chunks doubles, chunks + 1 floats
__global__ __launch_bounds__(1024) void mlstm_gates_kernel(const ps_seq_step *step, long long m_off, const float *iraw, const float *fraw, long long ldb, float cap, int H, int T,
                                                           int chunks, sd_gates G, float *mt) {
    extern __shared__ double gl[];
    double *cend = gl, *xmax = gl + chunks;
    float *ms = (float *)(xmax + chunks);
    const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    auto walk = [&](int k, double &c, double &x, double &top) { // the running sum, i - c and its running maximum at this lane's token of chunk k
        const int t = k * SD_Q + lane;
        const float li = t < T ? sd_capped(iraw[(long long)t * ldb + h], cap) : -INFINITY;
        c = t < T ? (double)sd_log_sigmoid(sd_capped(fraw[(long long)t * ldb + h], cap)) : 0.0;
#pragma unroll
        for (int o = 1; o < SD_Q; o <<= 1) {
            const double y = __shfl_up(c, o, 64);
            if (lane >= o) c += y;
        }
        x = (double)li - c;
        top = x;
#pragma unroll
        for (int o = 1; o < SD_Q; o <<= 1) {
            const double y = __shfl_up(top, o, 64);
            if (lane >= o) top = fmax(top, y);
        }
    };
    double c, x, top;
    for (int k = wave; k < chunks; k += nw) {
        walk(k, c, x, top);
        if (lane == SD_Q - 1) { cend[k] = c; xmax[k] = top; }
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        float m = step->state[m_off + h];
        for (int k = 0; k < chunks; k++) {
            ms[k] = m;
            m = (float)(cend[k] + fmax((double)m, xmax[k]));
        }
        ms[chunks] = m;
    }
    __syncthreads();
    for (int k = wave; k < chunks; k += nw) {
        walk(k, c, x, top);
        const double m_in = (double)ms[k];
        const float m = (float)(c + fmax(m_in, top));
        const double w = c - (double)m;
        const int t = k * SD_Q + lane;
        const long long at = (long long)h * chunks * SD_Q + t;
        G.u[at] = x;
        G.w[at] = w;
        G.lead[at] = expf((float)(w + m_in));
        G.tail[at] = expf((float)(cend[k] - (double)ms[k + 1] + x));
        if (t < T) mt[(long long)t * H + h] = m;
        if (lane == 0) G.dec[(long long)k * H + h] = expf((float)(cend[k] + m_in - (double)ms[k + 1]));
    }
}

// block (chunk, head, piece of the values); a wave takes units of 64 values x 32 state rows.  A lane's four value columns (two state rows) are neighbours: operand tile ii (jj) holds every
// fourth (second) one, and a result goes back to its place at the store.
template <bool LSTM>
__global__ __launch_bounds__(256) void ssd_state_kernel(const float *x, const float *B, long long ld, const float *dtraw, long long ldb, const float *a_log, const float *dt_bias, int H,
                                                        int G, int N, int P, int T, float *U, float *dec, sd_gates gates) {
    __shared__ double cs[SD_Q];
    __shared__ float dts[SD_Q], ws[SD_Q];
    const int h = blockIdx.y, t0 = blockIdx.x * SD_Q, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, lr = lane & 15, lq = lane >> 4;
    if constexpr (LSTM) {
        if (tid < SD_Q) ws[tid] = gates.tail[(long long)h * gridDim.x * SD_Q + t0 + tid];
    } else {
        sd_decays(dtraw, ldb, a_log, dt_bias, h, t0, T, cs, dts);
        if (tid < SD_Q) ws[tid] = expf((float)(cs[SD_Q - 1] - cs[tid])) * dts[tid];
        if (tid == 0) dec[(long long)blockIdx.x * H + h] = expf((float)cs[SD_Q - 1]);
    }
    __syncthreads();
    const float *xh = x + (long long)h * P, *Bh = B + (long long)(h / (H / G)) * N;
    float *Uh = U + ((long long)blockIdx.x * H + h) * (P + (LSTM ? 1 : 0)) * N;
    if constexpr (LSTM) { // the column of ones
        for (int n = tid; blockIdx.z == 0 && n < N; n += 256) {
            float a = 0.f;
#pragma unroll 16
            for (int s = 0; s < SD_Q; s++) a = fmaf(ws[s], Bh[(long long)(t0 + s < T ? t0 + s : T - 1) * ld + n], a);
            Uh[(long long)P * N + n] = a;
        }
    }
    const int nJ = (N + 31) / 32, units = (P + 63) / 64 * nJ;
    for (int u = wave + 4 * (int)blockIdx.z; u < units; u += 4 * (int)gridDim.z) {
        const int p = u / nJ * 64 + 4 * lr, n = u % nJ * 32 + 2 * lr;
        sd_f4 acc[4][2];
#pragma unroll
        for (int ii = 0; ii < 4; ii++)
#pragma unroll
            for (int jj = 0; jj < 2; jj++) acc[ii][jj] = sd_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int half = 0; half < 2; half++) {
            sd_f4 xv[8];
            sd_f2 bv[8];
#pragma unroll
            for (int k = 0; k < 8; k++) {
                const int s = half * 32 + 4 * k + lq, t = t0 + s < T ? t0 + s : T - 1;
                xv[k] = p < P ? *(const sd_f4 *)(xh + (long long)t * ld + p) : sd_f4{0.f, 0.f, 0.f, 0.f};
                bv[k] = n < N ? *(const sd_f2 *)(Bh + (long long)t * ld + n) : sd_f2{0.f, 0.f};
            }
#pragma unroll
            for (int k = 0; k < 8; k++) {
                const float w = ws[half * 32 + 4 * k + lq];
#pragma unroll
                for (int ii = 0; ii < 4; ii++)
#pragma unroll
                    for (int jj = 0; jj < 2; jj++) acc[ii][jj] = __builtin_amdgcn_mfma_f32_16x16x4f32(xv[k][ii] * w, bv[k][jj], acc[ii][jj], 0, 0, 0);
            }
        }
        if (n >= N) continue;
#pragma unroll
        for (int ii = 0; ii < 4; ii++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int pr = u / nJ * 64 + 4 * (4 * lq + i) + ii;
                if (pr < P) *(sd_f2 *)(Uh + (long long)pr * N + n) = sd_f2{acc[ii][0][i], acc[ii][1][i]};
            }
    }
}

// U[chunk] <- the state in front of the chunk; the slot's state <- the state behind the last one.  per_head: 16-byte pieces of a head's state
__global__ __launch_bounds__(256) void ssd_pass_kernel(const ps_seq_step *step, long long state_off, float *U, const float *dec, int H, long long per_head, int chunks) {
    const long long i = (long long)blockIdx.x * 256 + threadIdx.x, all = (long long)H * per_head;
    if (i >= all) return;
    const int h = (int)(i / per_head);
    sd_f4 *S0 = (sd_f4 *)(step->state + state_off) + i, *u = (sd_f4 *)U + i;
    sd_f4 S = *S0, next = u[0];
    for (int c = 0; c < chunks; c++) {
        const sd_f4 add = next;
        if (c + 1 < chunks) next = u[(long long)(c + 1) * all];
        u[(long long)c * all] = S;
        const float g = dec[(long long)c * H + h];
#pragma unroll
        for (int e = 0; e < 4; e++) S[e] = fmaf(g, S[e], add[e]);
    }
    *S0 = S;
}

// 16 rows (LDS, this lane's row lr at quarter lq) times one row of K numbers per lane (memory, at quarter lq): eight 16-byte pieces in flight, summed over a permutation of K
static __device__ __forceinline__ sd_f4 sd_dot(const float *qr, const float *kr, int K) {
    sd_f4 s = {0.f, 0.f, 0.f, 0.f};
    for (int g0 = 0; g0 < K; g0 += 128) {
        sd_f4 b[8];
#pragma unroll
        for (int u = 0; u < 8; u++) b[u] = g0 + 16 * u < K ? *(const sd_f4 *)(kr + g0 + 16 * u) : sd_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int u = 0; u < 8; u++)
            if (g0 + 16 * u < K) {
                const sd_f4 a = *(const sd_f4 *)(qr + g0 + 16 * u);
#pragma unroll
                for (int e = 0; e < 4; e++) s = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[u][e], s, 0, 0, 0);
            }
    }
    return s;
}
// block (chunk, head, piece of the values), a wave per 16 tokens.  Value columns in groups of 64, a lane's four tiles of a group are four neighbours.  NJ: tiles held (a piece is 16 NJ
// values; LSTM: C comes times qscale, and the first piece's block also makes nq, the product with the column of ones: n C plus the row sums of the masked products).
// dynamic LDS: 4 x (16 x (N + 4) + 16 x 17)
template <int NJ, bool LSTM>
__global__ __launch_bounds__(256) void ssd_out_kernel(const float *x, const float *B, const float *C, long long ld, const float *dtraw, long long ldb, const float *a_log,
                                                      const float *dt_bias, const float *skip, const float *Sin, int H, int G, int N, int Pall, int T, float *o, long long ldo,
                                                      sd_gates gates, float qscale, float *nq) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ double cs[SD_Q], us[SD_Q]; // (LSTM: w and u)
    __shared__ float dts[SD_Q];           // (LSTM: lead)
    const int h = blockIdx.y, t0 = blockIdx.x * SD_Q, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lq = lane >> 4, qld = N + 4;
    float *qs = lds + wave * (16 * qld + 16 * 17), *pt = qs + 16 * qld;
    const int w0 = t0 + wave * 16; // this wave's first token
    const int p0 = blockIdx.z * 16 * NJ, P = min(16 * NJ, Pall - p0); // this block's values
    const float *xh = x + (long long)h * Pall + p0, *Bh = B + (long long)(h / (H / G)) * N, *Ch = C + (long long)(h / (H / G)) * N;
    for (int r = 0; r < 16; r++) {
        const float *ct = Ch + (long long)(w0 + r < T ? w0 + r : T - 1) * ld;
        for (int c = 4 * lane; c < N; c += 256) {
            sd_f4 v = *(const sd_f4 *)(ct + c);
            if constexpr (LSTM) {
#pragma unroll
                for (int e = 0; e < 4; e++) v[e] *= qscale;
            }
            *(sd_f4 *)(qs + r * qld + c) = v;
        }
    }
    if constexpr (LSTM) {
        if (threadIdx.x < SD_Q) {
            const long long at = (long long)h * gridDim.x * SD_Q + t0 + threadIdx.x;
            cs[threadIdx.x] = gates.w[at];
            us[threadIdx.x] = gates.u[at];
            dts[threadIdx.x] = gates.lead[at];
        }
        __syncthreads();
    } else {
        sd_decays(dtraw, ldb, a_log, dt_bias, h, t0, T, cs, dts); // (with the block's barrier)
    }
    if (w0 >= T) return;
    const float *qr = qs + lr * qld + 4 * lq;
    sd_f4 acc[NJ];
    float lows[4] = {0.f, 0.f, 0.f, 0.f}; // LSTM: row 4 lq + i of nq, this lane's share
    {
        const float *Sh = Sin + ((long long)blockIdx.x * H + h) * (Pall + (LSTM ? 1 : 0)) * N + (long long)p0 * N;
        float e[4];
#pragma unroll
        for (int i = 0; i < 4; i++) e[i] = LSTM ? dts[wave * 16 + 4 * lq + i] : expf((float)cs[wave * 16 + 4 * lq + i]);
        if constexpr (LSTM) {
            if (blockIdx.z == 0) { // n C: row lr, a quarter of the numbers per lane
                const float *n = Sh + (long long)Pall * N + 4 * lq;
                float d = 0.f;
                for (int c = 0; c < N; c += 16) {
                    const sd_f4 a = *(const sd_f4 *)(qr + c), b = *(const sd_f4 *)(n + c);
#pragma unroll
                    for (int k = 0; k < 4; k++) d = fmaf(a[k], b[k], d);
                }
                d += __shfl_xor(d, 16, 64);
                d += __shfl_xor(d, 32, 64);
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const float r = __shfl(d, 4 * lq + i, 64) * e[i];
                    lows[i] = lr == 0 ? r : 0.f;
                }
            }
        }
#pragma unroll
        for (int j = 0; j < NJ; j++) {
            acc[j] = sd_f4{0.f, 0.f, 0.f, 0.f};
            if (64 * (j / 4) >= P) continue; // (uniform)
            const int p = 64 * (j / 4) + 4 * lr + j % 4;
            const sd_f4 s = sd_dot(qr, Sh + (long long)(p < P ? p : P - 1) * N + 4 * lq, N);
#pragma unroll
            for (int i = 0; i < 4; i++) acc[j][i] = s[i] * e[i];
        }
    }
    for (int st = 0; st <= wave; st++) {
        const int s = st * 16 + lr;
        const sd_f4 g = sd_dot(qr, Bh + (long long)(t0 + s < T ? t0 + s : T - 1) * ld + 4 * lq, N);
        sd_f4 xv[NJ / 4][4];
#pragma unroll
        for (int k = 0; k < 4; k++) {
            const int t = t0 + st * 16 + 4 * k + lq;
#pragma unroll
            for (int J = 0; J < NJ / 4; J++)
                xv[J][k] = 64 * J + 4 * lr < P ? *(const sd_f4 *)(xh + (long long)(t < T ? t : T - 1) * ld + 64 * J + 4 * lr) : sd_f4{0.f, 0.f, 0.f, 0.f};
        }
        const double c = LSTM ? us[s] : cs[s];
        const float dt = dts[s];
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = wave * 16 + 4 * lq + i;
            float pv = 0.f;
            if (s <= t) pv = LSTM ? g[i] * expf((float)(cs[t] + c)) : g[i] * (expf((float)(cs[t] - c)) * dt);
            pt[(4 * lq + i) * 17 + lr] = pv;
            if constexpr (LSTM) lows[i] += pv;
        }
        __builtin_amdgcn_wave_barrier();
        float pa[4];
#pragma unroll
        for (int k = 0; k < 4; k++) pa[k] = pt[lr * 17 + 4 * k + lq];
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int J = 0; J < NJ / 4; J++)
            if (64 * J < P) {
#pragma unroll
                for (int jj = 0; jj < 4; jj++)
#pragma unroll
                    for (int k = 0; k < 4; k++) acc[4 * J + jj] = __builtin_amdgcn_mfma_f32_16x16x4f32(pa[k], xv[J][k][jj], acc[4 * J + jj], 0, 0, 0);
            }
    }
    if constexpr (LSTM) {
        if (blockIdx.z == 0) {
#pragma unroll
            for (int i = 0; i < 4; i++) {
                float a = lows[i];
#pragma unroll
                for (int x = 1; x < 16; x <<= 1) a += __shfl_xor(a, x, 64);
                if (lr == 0 && w0 + 4 * lq + i < T) nq[(long long)(w0 + 4 * lq + i) * H + h] = a;
            }
        }
    }
    const float sk = LSTM ? 0.f : skip[h];
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int t = w0 + 4 * lq + i;
        if (t >= T) continue;
#pragma unroll
        for (int J = 0; J < NJ / 4; J++) {
            const int c = 64 * J + 4 * lr;
            if (c >= P) continue;
            sd_f4 r = {acc[4 * J][i], acc[4 * J + 1][i], acc[4 * J + 2][i], acc[4 * J + 3][i]};
            if constexpr (!LSTM) {
                const sd_f4 xt = *(const sd_f4 *)(xh + (long long)t * ld + c);
#pragma unroll
                for (int e = 0; e < 4; e++) r[e] = fmaf(sk, xt[e], r[e]);
            }
            *(sd_f4 *)(o + (long long)t * ldo + (long long)h * Pall + p0 + c) = r;
        }
    }
}

// sizes the chunked form takes: 16-byte pieces of the state's rows (N a multiple of 16) and of the values (P of 4, at most 128)
bool psk_ssd_chunked_ok(int N, int P) { return N % 16 == 0 && N <= 256 && P % 4 == 0 && P <= 128; }
size_t psk_ssd_chunked_scratch(int H, int N, int P, int T) {
    const size_t chunks = (size_t)(T + SD_Q - 1) / SD_Q;
    return chunks * ((size_t)H * P * N + (size_t)(H + 3) / 4 * 4) * 4;
}
void psk_ssd_chunked(hipStream_t st, const ps_seq_step *step, int64_t state_off, const float *x, const float *B, const float *C, int64_t ld, const float *dtraw, int64_t ldb,
                     const float *a_log, const float *dt_bias, const float *skip, int H, int G, int N, int P, int T, float *scratch, float *o, int64_t ldo) {
    const int chunks = (T + SD_Q - 1) / SD_Q;
    float *U = scratch, *dec = U + (size_t)chunks * H * P * N;
    hipLaunchKernelGGL(ssd_state_kernel<false>, dim3(chunks, H), dim3(256), 0, st, x, B, (long long)ld, dtraw, (long long)ldb, a_log, dt_bias, H, G, N, P, T, U, dec, sd_gates{});
    const long long per_head = (long long)P * N / 4;
    hipLaunchKernelGGL(ssd_pass_kernel, dim3((unsigned)((per_head * H + 255) / 256)), dim3(256), 0, st, step, (long long)state_off, U, dec, H, per_head, chunks);
    const size_t lds = (size_t)4 * (16 * (N + 4) + 16 * 17) * 4;
    static unsigned long long mask = 0;
    if (ps_first_on_device(&mask)) {
        (void)hipFuncSetAttribute((const void *)ssd_out_kernel<4, false>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
        (void)hipFuncSetAttribute((const void *)ssd_out_kernel<8, false>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    }
    const auto kernel = P <= 64 ? ssd_out_kernel<4, false> : ssd_out_kernel<8, false>;
    hipLaunchKernelGGL(kernel, dim3(chunks, H), dim3(256), lds, st, x, B, C, (long long)ld, dtraw, (long long)ldb, a_log, dt_bias, skip, U, H, G, N, P, T, o, (long long)ldo,
                       sd_gates{}, 1.f, nullptr);
}

// sizes: 16-byte pieces of q, k and the state's rows (d a multiple of 16) and of the values (dv of 4, any number of them: pieces of 128)
bool psk_mlstm_chunked_ok(int d, int dv) { return d % 16 == 0 && d <= 256 && dv % 4 == 0; }
size_t psk_mlstm_chunked_scratch(int H, int d, int dv, int T) {
    const size_t chunks = (size_t)(T + SD_Q - 1) / SD_Q;
    return chunks * ((size_t)H * (dv + 1) * d * 4 + (size_t)H * SD_Q * (8 + 8 + 4 + 4) + (size_t)(H + 3) / 4 * 16);
}
void psk_mlstm_chunked(hipStream_t st, const ps_seq_step *step, int64_t state_off, int64_t m_off, const float *q, const float *k, const float *v, int64_t ld, const float *iraw,
                       const float *fraw, int64_t ldb, float cap, int H, int d, int dv, int T, float *scratch, float *o, int64_t ldo, float *nq, float *mt) {
    const int chunks = (T + SD_Q - 1) / SD_Q;
    const size_t per = (size_t)chunks * H * SD_Q;
    float *U = scratch;
    sd_gates G;
    G.u = (double *)(U + (size_t)chunks * H * (dv + 1) * d); // (d a multiple of 16: 8-byte aligned)
    G.w = G.u + per;
    G.lead = (float *)(G.w + per);
    G.tail = G.lead + per;
    G.dec = G.tail + per;
    hipLaunchKernelGGL(mlstm_gates_kernel, dim3(H), dim3(64 * (chunks < 16 ? chunks : 16)), (size_t)chunks * 16 + (size_t)(chunks + 1) * 4, st, step, (long long)m_off, iraw, fraw,
                       (long long)ldb, cap, H, T, chunks, G, mt);
    hipLaunchKernelGGL(ssd_state_kernel<true>, dim3(chunks, H, (unsigned)std::max(1, ((dv + 63) / 64 * ((d + 31) / 32) + 3) / 4)), dim3(256), 0, st, v, k, (long long)ld, nullptr, 0ll, nullptr, nullptr, H, H, d, dv, T, U, nullptr, G);
    const long long per_head = (long long)(dv + 1) * d / 4;
    hipLaunchKernelGGL(ssd_pass_kernel, dim3((unsigned)((per_head * H + 255) / 256)), dim3(256), 0, st, step, (long long)state_off, U, G.dec, H, per_head, chunks);
    const size_t lds = (size_t)4 * (16 * (d + 4) + 16 * 17) * 4;
    static unsigned long long mask = 0;
    if (ps_first_on_device(&mask)) {
        (void)hipFuncSetAttribute((const void *)ssd_out_kernel<4, true>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
        (void)hipFuncSetAttribute((const void *)ssd_out_kernel<8, true>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    }
    // pieces of 64 values where pieces of 128 would leave CUs without a block
    const bool small = dv <= 64 || (long long)chunks * H * ((dv + 127) / 128) < 512;
    const auto kernel = small ? ssd_out_kernel<4, true> : ssd_out_kernel<8, true>;
    hipLaunchKernelGGL(kernel, dim3(chunks, H, small ? (dv + 63) / 64 : (dv + 127) / 128), dim3(256), lds, st, v, k, q, (long long)ld, nullptr, 0ll, nullptr, nullptr, nullptr, U, H, H, d, dv, T, o,
                       (long long)ldo, G, 1.f / sqrtf((float)d), nq);
}
