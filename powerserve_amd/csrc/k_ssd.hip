// The state-space recurrence of the layer-list models (PS_MIX_SSD) for a portion of tokens, in CHUNKS on the fp32 matrix cores.  Per head, with dt_t = softplus(dtraw + dt_bias),
// a_t = -exp(a_log) dt_t and c_t the running sum of a over a chunk of 64 tokens, the token-by-token scan (k_seqmix.hip) is the same as
//   U     = sum_s exp(c_end - c_s) dt_s x_s B_s^T               what a chunk adds to the state                  ssd_state_kernel, all chunks at once
//   S_in  <- exp(c_end) S_in + U                                the state in front of every chunk               ssd_pass_kernel, an element per lane, chunk after chunk
//   y_t   = exp(c_t) S_in C_t + sum_(s <= t) exp(c_t - c_s) dt_s (C_t . B_s) x_s + skip x_t                     ssd_out_kernel, all chunks at once
// Everything is fp32 (v_mfma_f32_16x16x4_f32); the running sums are kept in double, so that a difference of two of them is as good as its own size asks for.  Exponents are
// never positive.  x [T][H P], B and C [T][G N] share a row stride; the state is [H][P][N].
#include "ps_seq.h"

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

// block (chunk, head); a wave takes units of 64 values x 32 state rows.  A lane's four value columns (two state rows) are neighbours: operand tile ii (jj) holds every
// fourth (second) one, and a result goes back to its place at the store.
__global__ __launch_bounds__(256) void ssd_state_kernel(const float *x, const float *B, long long ld, const float *dtraw, long long ldb, const float *a_log, const float *dt_bias, int H,
                                                        int G, int N, int P, int T, float *U, float *dec) {
    __shared__ double cs[SD_Q];
    __shared__ float dts[SD_Q], ws[SD_Q];
    const int h = blockIdx.y, t0 = blockIdx.x * SD_Q, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, lr = lane & 15, lq = lane >> 4;
    sd_decays(dtraw, ldb, a_log, dt_bias, h, t0, T, cs, dts);
    if (tid < SD_Q) ws[tid] = expf((float)(cs[SD_Q - 1] - cs[tid])) * dts[tid];
    if (tid == 0) dec[(long long)blockIdx.x * H + h] = expf((float)cs[SD_Q - 1]);
    __syncthreads();
    const float *xh = x + (long long)h * P, *Bh = B + (long long)(h / (H / G)) * N;
    float *Uh = U + ((long long)blockIdx.x * H + h) * P * N;
    const int nJ = (N + 31) / 32, units = (P + 63) / 64 * nJ;
    for (int u = wave; u < units; u += 4) {
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
// block (chunk, head), a wave per 16 tokens.  Value columns in groups of 64, a lane's four tiles of a group are four neighbours.  NJ: tiles held (P <= 16 NJ).
// dynamic LDS: 4 x (16 x (N + 4) + 16 x 17)
template <int NJ>
__global__ __launch_bounds__(256) void ssd_out_kernel(const float *x, const float *B, const float *C, long long ld, const float *dtraw, long long ldb, const float *a_log,
                                                      const float *dt_bias, const float *skip, const float *Sin, int H, int G, int N, int P, int T, float *o, long long ldo) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ double cs[SD_Q];
    __shared__ float dts[SD_Q];
    const int h = blockIdx.y, t0 = blockIdx.x * SD_Q, wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lq = lane >> 4, qld = N + 4;
    float *qs = lds + wave * (16 * qld + 16 * 17), *pt = qs + 16 * qld;
    const int w0 = t0 + wave * 16; // this wave's first token
    const float *xh = x + (long long)h * P, *Bh = B + (long long)(h / (H / G)) * N, *Ch = C + (long long)(h / (H / G)) * N;
    for (int r = 0; r < 16; r++) {
        const float *ct = Ch + (long long)(w0 + r < T ? w0 + r : T - 1) * ld;
        for (int c = 4 * lane; c < N; c += 256) *(sd_f4 *)(qs + r * qld + c) = *(const sd_f4 *)(ct + c);
    }
    sd_decays(dtraw, ldb, a_log, dt_bias, h, t0, T, cs, dts); // (with the block's barrier)
    if (w0 >= T) return;
    const float *qr = qs + lr * qld + 4 * lq;
    sd_f4 acc[NJ];
    {
        const float *Sh = Sin + ((long long)blockIdx.x * H + h) * P * N;
        float e[4];
#pragma unroll
        for (int i = 0; i < 4; i++) e[i] = expf((float)cs[wave * 16 + 4 * lq + i]);
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
        const double c = cs[s];
        const float dt = dts[s];
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = wave * 16 + 4 * lq + i;
            pt[(4 * lq + i) * 17 + lr] = s <= t ? g[i] * (expf((float)(cs[t] - c)) * dt) : 0.f;
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
    const float sk = skip[h];
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int t = w0 + 4 * lq + i;
        if (t >= T) continue;
#pragma unroll
        for (int J = 0; J < NJ / 4; J++) {
            const int c = 64 * J + 4 * lr;
            if (c >= P) continue;
            const sd_f4 xt = *(const sd_f4 *)(xh + (long long)t * ld + c);
            sd_f4 r;
#pragma unroll
            for (int e = 0; e < 4; e++) r[e] = fmaf(sk, xt[e], acc[4 * J + e][i]);
            *(sd_f4 *)(o + (long long)t * ldo + (long long)h * P + c) = r;
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
    hipLaunchKernelGGL(ssd_state_kernel, dim3(chunks, H), dim3(256), 0, st, x, B, (long long)ld, dtraw, (long long)ldb, a_log, dt_bias, H, G, N, P, T, U, dec);
    const long long per_head = (long long)P * N / 4;
    hipLaunchKernelGGL(ssd_pass_kernel, dim3((unsigned)((per_head * H + 255) / 256)), dim3(256), 0, st, step, (long long)state_off, U, dec, H, per_head, chunks);
    const size_t lds = (size_t)4 * (16 * (N + 4) + 16 * 17) * 4;
    static unsigned long long mask = 0;
    if (ps_first_on_device(&mask)) {
        (void)hipFuncSetAttribute((const void *)ssd_out_kernel<4>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
        (void)hipFuncSetAttribute((const void *)ssd_out_kernel<8>, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    }
    const auto kernel = P <= 64 ? ssd_out_kernel<4> : ssd_out_kernel<8>;
    hipLaunchKernelGGL(kernel, dim3(chunks, H), dim3(256), lds, st, x, B, C, (long long)ld, dtraw, (long long)ldb, a_log, dt_bias, skip, U, H, G, N, P, T, o, (long long)ldo);
}
