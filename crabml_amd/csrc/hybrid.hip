// hybrid.hip -- the hybrid decoder (crabml_hip_hybrid_*): host side.  Context, weight packing, the sequences' state slabs, the decode
// step as a captured graph, the prompt pass, the C entry points.  Kernels: hybrid_step.hpp, hybrid_rows.hpp, hybrid_latent.hpp, gemv_bf16.hpp,
// gemm_bf16.hip.
#include <cmath>
#include <memory>

#include "dequant.hpp"
#include "hybrid_latent.hpp"
#include "hybrid_rows.hpp"
#include "hybrid_step.hpp"
#include "lazy.hpp"

using namespace crabml_hip;

namespace {

struct Connection {  // a sublayer between the residual streams
  float *coef = nullptr, *in = nullptr;
};
struct Layer {
  AttnGeom at;
  LatGeom la;
  LinGeom li;
  Connection hc[2];  // mixer, feed-forward
  bool glu = false;
  float *bias_in = nullptr, *bias_o = nullptr;
  int n_in = 0, ldc = 0, lin_off = 0, ff = 0, ldu = 0, splits = 0, head_blocks = 0;
  ActRanges act;
  unsigned short *w_in = nullptr, *w_o = nullptr, *w_up = nullptr, *w_down = nullptr;
  float *norm1 = nullptr, *norm2 = nullptr, *xielu = nullptr;
};
struct Run {  // one execution of a layer: in a loop, every time is a run of its own
  int layer = 0;
  RunState rs;
  bool add_emb = false;            // what is added to x in front of it
  const float* add_vec = nullptr;
};
struct Seq {
  bool open = false;
  char* slab = nullptr;
  size_t cap = 0;
  size_t len = 0;
};
// profiling stages (crabml_hip_prof_*): decode 11 .., prompt pass 21 ..
// (ROWS: row kernels around a mixer, in a decode step the latent values; LAT: latent queries, in a pass the keys and values)
enum { ST_IN = 1, ST_MIX = 2, ST_OUT = 3, ST_UP = 4, ST_DOWN = 5, ST_HEAD = 6, ST_LIN = 7, ST_ROWS = 8, ST_LAT = 9, ST_STEP = 10, ST_PASS = 20 };

constexpr size_t LOGIT_ROWS = 256;  // rows of logits a pass keeps on the device at a time
constexpr int META_SLOTS = 4;

}  // namespace

struct crabml_hip_hybrid {
  crabml_hip_device* dev = nullptr;
  crabml_hip_hybrid_config_t cfg{};
  bool f32 = false;
  int planes = 1;
  int width = 0, vocab = 0, ldx = 0, n_sq = 0;
  std::vector<Layer> layers;
  std::vector<Run> runs;
  std::vector<Seq> seqs;
  size_t slab_bytes = 0;
  unsigned short *embed = nullptr, *head = nullptr;
  float *loop_step = nullptr, *final_norm = nullptr, *ones = nullptr;
  int streams = 0;  // 0: one residual row, norms with a single gain; else gains per element
  double* freq = nullptr;
  bool keep_emb = false;
  // decode step
  StepSeq* st_seq = nullptr;
  int* st_count = nullptr;
  float *st_x = nullptr, *st_emb = nullptr, *st_proj = nullptr, *st_cat = nullptr, *st_u = nullptr, *st_ss = nullptr, *st_part = nullptr, *st_logits = nullptr;
  float *st_in = nullptr, *st_vk = nullptr, *st_q = nullptr, *st_lpart = nullptr;  // streams: what the next linear reads; kept values; latent queries, partials
  int ld_vk = 0, ld_kv = 0, ld_lat = 0, ld_rot = 0;
  size_t hist = 0;  // earlier positions a latent layer can see
  unsigned* st_tick = nullptr;
  unsigned* st_out = nullptr;
  size_t st_out_cap = 0;
  float* am_val = nullptr;
  int* am_idx = nullptr;
  int ld_proj = 0, ld_cat = 0, ld_u = 0;
  StepSeq* h_seq = nullptr;  // pinned ring of META_SLOTS * HYB_STEP_ROWS
  int h_seq_next = 0;
  std::map<int, std::pair<hipGraph_t, hipGraphExec_t>> graphs;  // key: rows * 2 + sampler
  // prompt pass (allocated on first use)
  size_t rows_cap = 0, hist_cap = 0, meta_bytes = 0;
  char *meta = nullptr, *h_meta = nullptr;
  int h_meta_next = 0;
  float *pf_x = nullptr, *pf_emb = nullptr, *pf_lin = nullptr, *pf_sq = nullptr, *pf_gsq = nullptr, *pf_logits = nullptr;
  unsigned short *pf_xp = nullptr, *pf_cat = nullptr, *pf_u = nullptr, *pf_gp = nullptr;
  void *pf_proj = nullptr, *pf_vk = nullptr, *pf_rot = nullptr, *pf_kv = nullptr;
  unsigned short* pf_lat = nullptr;
  GemmScratch pf_scratch;
  hipStream_t side = nullptr;  // the linear branch of a long pass, beside the softmax branch
  hipEvent_t fork = nullptr, join = nullptr;
  std::vector<std::pair<void*, size_t>> allocs;
};

namespace {

typedef crabml_hip_hybrid Ctx;

int dalloc(Ctx* c, size_t bytes, void** out, bool clear = true) {
  size_t cap = 0;
  if (bytes < 16) bytes = 16;
  CH_TRY(pool_alloc(c->dev, bytes, out, &cap));
  c->allocs.push_back({*out, cap});
  if (clear) CH_HIP(c->dev, hipMemsetAsync(*out, 0, bytes, c->dev->stream));
  return 0;
}
template <typename T>
int dalloc_n(Ctx* c, size_t n, T** out) {
  return dalloc(c, n * sizeof(T), (void**)out);
}
int up(size_t v, size_t a) { return (int)align_up(v, a); }

// ---- weight packing -----------------------------------------------------------------------------------------------------------------
// row r -> row0 + r with every group of rg rows widened to rgp; columns the same (head widths padded; the gaps stay zero).  The rows are
// the `rg` from `so` on of every group of sg source rows.
__global__ __launch_bounds__(256) void k_pack_matrix(const unsigned short* __restrict__ src, int m, int k, unsigned short* __restrict__ dst, size_t ldd,
                                                     int row0, int rg, int rgp, int col0, int cg, int cgp, int sg, int so) {
  const int r = blockIdx.y;
  const unsigned short* x = src + (size_t)(r / rg * sg + so + r % rg) * k;
  unsigned short* d = dst + (size_t)(row0 + r / rg * rgp + r % rg) * ldd + col0;
  for (int c = blockIdx.x * 256 + threadIdx.x; c < k; c += gridDim.x * 256) d[c / cg * cgp + c % cg] = x[c];
}
// [heads][dim][k] -> [heads][kp][dimp]
__global__ __launch_bounds__(256) void k_pack_transposed(const unsigned short* __restrict__ src, int dim, int k, unsigned short* __restrict__ dst, int kp, int dimp) {
  const int h = blockIdx.z, d = blockIdx.y;
  const unsigned short* x = src + ((size_t)h * dim + d) * k;
  for (int c = blockIdx.x * 256 + threadIdx.x; c < k; c += gridDim.x * 256) dst[((size_t)h * kp + c) * dimp + d] = x[c];
}
__global__ __launch_bounds__(256) void k_pack_vector(const char* __restrict__ src, int dtype, size_t off_scale, int n, float* __restrict__ dst, int g, int gp,
                                                     float plus, int wrap) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < n) dst[i / g * gp + i % g] = dequant_elem(src, dtype, off_scale, i % wrap) + plus;
}
// a connection's raw numbers -> rows of StreamMix::coef
__global__ void k_pack_connection(const float* __restrict__ mix, const float* __restrict__ out, int n, float* __restrict__ coef) {
  for (int t = 0; t < n; t++) {
    for (int s = 0; s < HC_MAX; s++) coef[t * HC_ROW + s] = s < n ? mix[s * n + t] : 0.f;
    coef[t * HC_ROW + HC_MAX] = out[t];
  }
}
__global__ void k_xielu_consts(const float* __restrict__ raw, float* __restrict__ out) {
  auto softplus = [](float z) { return log1pf(expf(-fabsf(z))) + fmaxf(z, 0.f); };
  out[0] = softplus(raw[0]);
  out[1] = 0.5f + softplus(raw[1]);
}

int pack_matrix(Ctx* c, const crabml_hip_buf* b, const char* what, size_t m, size_t k, unsigned short* dst, size_t ldd, size_t row0, size_t rg, size_t rgp,
                size_t col0 = 0, size_t cg = 0, size_t cgp = 0, size_t sg = 0, size_t so = 0) {
  if (sg == 0) sg = rg;
  const size_t rows = rg ? m / rg * sg : m;  // (m: the rows that are taken)
  if (!b || b->dtype != CRABML_HIP_BF16 || b->n_elems != rows * k || b->dev != c->dev)
    CH_BAIL(c->dev, CRABML_HIP_BAD_INPUT, "hybrid: %s must be a bfloat16 matrix of %zu x %zu", what, rows, k);
  k_pack_matrix<<<dim3((unsigned)std::min<size_t>((k + 255) / 256, 64), (unsigned)m), 256, 0, c->dev->stream>>>(
      (const unsigned short*)b->ptr, (int)m, (int)k, dst, ldd, (int)row0, (int)rg, (int)rgp, (int)col0, (int)(cg ? cg : k), (int)(cg ? cgp : k), (int)sg, (int)so);
  CH_HIP(c->dev, hipGetLastError());
  return 0;
}
// n numbers into dst, every group of g widened to gp
int pack_into(Ctx* c, const crabml_hip_buf* b, const char* what, size_t n, float* dst, size_t g = 0, size_t gp = 0, float plus = 0.f) {
  if (!b || b->n_elems != n || b->dev != c->dev) CH_BAIL(c->dev, CRABML_HIP_BAD_INPUT, "hybrid: %s must hold %zu numbers", what, n);
  if (g == 0) g = gp = n;
  k_pack_vector<<<(unsigned)((n + 255) / 256), 256, 0, c->dev->stream>>>((const char*)b->ptr, (int)b->dtype, b->wl.off_scale, (int)n, dst, (int)g, (int)gp, plus, (int)n);
  CH_HIP(c->dev, hipGetLastError());
  return 0;
}
int pack_vector(Ctx* c, const crabml_hip_buf* b, const char* what, size_t n, float** out, size_t g = 0, size_t gp = 0) {
  if (g == 0) g = gp = n;
  CH_TRY(dalloc_n(c, n / g * gp, out));
  return pack_into(c, b, what, n, *out, g, gp);
}
// an RMS norm's gain: one number, or (streams) one per element of a padded row, wherever the design has a single one
int pack_norm(Ctx* c, const crabml_hip_buf* b, const char* what, float** out) {
  const float plus = c->cfg.flags & CRABML_HIP_HYBRID_NORM_ONE_PLUS ? 1.f : 0.f;
  const size_t n = c->cfg.flags & CRABML_HIP_HYBRID_NORM_VECTOR ? (size_t)c->width : 1;
  if (!b || b->n_elems != n || b->dev != c->dev) CH_BAIL(c->dev, CRABML_HIP_BAD_INPUT, "hybrid: %s must hold %zu numbers", what, n);
  const size_t m = c->streams ? (size_t)c->width : 1;
  CH_TRY(dalloc_n(c, c->streams ? align_up(m, 64) : m, out));
  k_pack_vector<<<(unsigned)((m + 255) / 256), 256, 0, c->dev->stream>>>((const char*)b->ptr, (int)b->dtype, b->wl.off_scale, (int)m, *out, (int)m, (int)m, plus, (int)n);
  CH_HIP(c->dev, hipGetLastError());
  return 0;
}
int pack_connection(Ctx* c, const crabml_hip_buf* in, const crabml_hip_buf* out, const crabml_hip_buf* mix, Connection& h) {
  const size_t n = (size_t)c->streams;
  float *m = nullptr, *o = nullptr;
  if (!c->cfg.streams) {  // a plain residual: one stream that keeps itself
    h.in = o = m = c->ones;
  } else {
    CH_TRY(dalloc_n(c, HC_MAX, &h.in));
    CH_TRY(pack_into(c, in, "a connection's input weights", n, h.in));
    CH_TRY(pack_vector(c, out, "a connection's output weights", n, &o));
    CH_TRY(pack_vector(c, mix, "a connection's mixing matrix", n * n, &m));
  }
  CH_TRY(dalloc_n(c, HC_MAX * HC_ROW, &h.coef));
  k_pack_connection<<<1, 1, 0, c->dev->stream>>>(m, o, (int)n, h.coef);
  CH_HIP(c->dev, hipGetLastError());
  return 0;
}
// rows of a weight matrix: padded to 256 so that any tile of the GEMM reads inside it
int alloc_matrix(Ctx* c, size_t rows, size_t ld, unsigned short** out) { return dalloc_n(c, align_up(rows, 256) * ld, out); }

int build_layer(Ctx* c, const crabml_hip_hybrid_layer_t& s, Layer& L) {
  crabml_hip_device* dev = c->dev;
  const size_t W = (size_t)c->width, H = s.attn_heads, Hl = s.lin_heads, rank = s.attn_latent, rot = rank ? s.attn_rot : 0;
  const size_t G = rank ? H : s.attn_kv_heads;
  if (!H && !Hl) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: a layer needs a mixer");
  if (H && (!G || H % G || !s.attn_dim || !s.attn_vdim || s.attn_dim > 256 || s.attn_vdim > 256))
    CH_BAIL(dev, H && G && H % G == 0 ? CRABML_HIP_NOT_IMPLEMENTED : CRABML_HIP_BAD_INPUT, "hybrid: attention of %zu / %zu heads of %zu / %zu (at most 256 wide)", H, G,
            s.attn_dim, s.attn_vdim);
  const size_t dimp = align_up(s.attn_dim, 8), rotp = align_up(rot, 8), rankp = align_up(rank, 8);
  if (H && rank && (rot % 2 || dimp + rotp > 256 || rankp + rotp > LAT_MAX_ROW || !(s.attn_rot_base > 0 || !rot)))
    CH_BAIL(dev, CRABML_HIP_NOT_IMPLEMENTED, "hybrid: latent attention of rank %zu, heads of %zu + %zu rotated (rows at most %d, heads at most 256 wide, pairs rotated)", rank,
            s.attn_dim, rot, LAT_MAX_ROW);
  if (H && rank && (s.attn_gate || s.attn_sink || s.attn_bias_amp || s.attn_q_norm || s.attn_k_norm || s.attn_vmix || s.attn_q_bias || s.attn_k_bias || s.attn_v_bias || Hl))
    CH_BAIL(dev, CRABML_HIP_NOT_IMPLEMENTED, "hybrid: latent attention has no gate, sink, distance bias, query or key norm, value mixing or input biases, and no branch beside it");
  if (s.attn_chunk && s.attn_window) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: attention inside chunks or a window, not both");
  if (Hl && (!s.lin_dim || !s.lin_vdim || s.lin_dim > 256 || !s.lin_decay))
    CH_BAIL(dev, CRABML_HIP_NOT_IMPLEMENTED, "hybrid: linear attention of %zu heads of %zu / %zu (keys at most 256 wide, decay given)", Hl, s.lin_dim, s.lin_vdim);
  const size_t D = dimp + rotp, V = align_up(s.attn_vdim, 8), Dl = align_up(s.lin_dim, 8), Vl = align_up(s.lin_vdim, 8);
  size_t col = 0;
  auto take = [&](size_t n) {
    const size_t at = col;
    col += n;
    return (int)at;
  };
  AttnGeom& a = L.at;
  LinGeom& l = L.li;
  // columns of the projected row: raw q k v | sigmoid gate | silu q k v | sigmoid gate
  if (H) {
    a.H = (int)H;
    a.G = (int)G;
    a.D = (int)D;
    a.V = (int)V;
    const size_t limit = s.attn_window ? s.attn_window : s.attn_chunk;
    const size_t span = limit && limit < ((size_t)1 << 30) ? limit : (size_t)1 << 30;
    a.span = (int)span;
    a.window = s.attn_window != 0;
    a.rows = (int)std::min(span, c->cfg.seq_len);
    a.eps = c->cfg.norm_eps;
    a.scale = s.attn_score_scale;
    a.out_scale = s.attn_out_scale;
    a.cq = take(H * D);
    if (rank) {
      L.la.cc = take(rankp);
      L.la.cr = take(rotp);
    } else {
      a.ck = take(G * D);
      a.cv = take(G * V);
    }
  }
  L.act.end[0] = (int)col;
  if (H && s.attn_gate) {
    a.gate = s.attn_gate->n_elems == H * W && s.attn_vdim != 1 ? GATE_HEAD : GATE_ELEMENT;
    a.cg = a.gate == GATE_HEAD ? take(align_up(H, 8)) : take(H * V);
  }
  L.act.end[1] = (int)col;
  L.act.kind[1] = ACT_SIGMOID;
  if (Hl) {
    l.H = (int)Hl;
    l.D = (int)Dl;
    l.V = (int)Vl;
    l.v_true = (int)s.lin_vdim;
    l.out_scale = s.lin_out_scale;
    l.slices = (int)((Vl + LIN_SLICE - 1) / LIN_SLICE);
    l.cq = take(Hl * Dl);
    l.ck = take(Hl * Dl);
    l.cv = take(Hl * Vl);
  }
  L.act.end[2] = (int)col;
  L.act.kind[2] = ACT_SILU;
  if (Hl) l.cg = take(Hl * Vl);
  L.act.end[3] = (int)col;
  L.act.kind[3] = ACT_SIGMOID;
  L.n_in = (int)col;
  L.lin_off = up(H * V, 64);
  L.ldc = L.lin_off + up(Hl * Vl, 64);
  L.ff = (int)s.ff;
  L.ldu = up(s.ff, 64);
  L.splits = H && !rank ? (a.rows + MIX_KEYS - 1) / MIX_KEYS : 0;
  L.head_blocks = H && !rank ? (int)((H / G + MIX_HEADS - 1) / MIX_HEADS) : 0;
  const size_t ldw = (size_t)c->ldx;
  CH_TRY(alloc_matrix(c, col, ldw, &L.w_in));
  CH_TRY(alloc_matrix(c, W, (size_t)L.ldc, &L.w_o));
  if (H && (s.attn_q_bias || s.attn_k_bias || s.attn_v_bias)) {
    CH_TRY(dalloc_n(c, col, &L.bias_in));
    if (s.attn_q_bias) CH_TRY(pack_into(c, s.attn_q_bias, "attn_q_bias", H * s.attn_dim, L.bias_in + a.cq, s.attn_dim, D));
    if (s.attn_k_bias) CH_TRY(pack_into(c, s.attn_k_bias, "attn_k_bias", G * s.attn_dim, L.bias_in + a.ck, s.attn_dim, D));
    if (s.attn_v_bias) CH_TRY(pack_into(c, s.attn_v_bias, "attn_v_bias", G * s.attn_vdim, L.bias_in + a.cv, s.attn_vdim, V));
  }
  if (s.attn_o_bias) {
    if (!c->streams) CH_BAIL(dev, CRABML_HIP_NOT_IMPLEMENTED, "hybrid: an output bias goes with norms of a gain per element or with residual streams");
    CH_TRY(dalloc_n(c, align_up(W, 64), &L.bias_o));
    CH_TRY(pack_into(c, s.attn_o_bias, "attn_o_bias", W, L.bias_o));
  }
  if (H && rank) {
    LatGeom& la = L.la;
    la.rank = (int)rankp;
    la.dim = (int)dimp;
    la.rot = (int)rotp;
    la.rank_true = (int)rank;
    la.ldl = up(rank, 64);
    CH_TRY(pack_matrix(c, s.attn_q, "attn_q", H * s.attn_dim, W, L.w_in, ldw, a.cq, s.attn_dim, D, 0, 0, 0, s.attn_dim + rot, 0));
    if (rot) CH_TRY(pack_matrix(c, s.attn_q, "attn_q", H * rot, W, L.w_in, ldw, a.cq + dimp, rot, D, 0, 0, 0, s.attn_dim + rot, s.attn_dim));
    CH_TRY(pack_matrix(c, s.attn_latent_down, "attn_latent_down", rank, W, L.w_in, ldw, la.cc, rank, rankp, 0, 0, 0, rank + rot, 0));
    if (rot) CH_TRY(pack_matrix(c, s.attn_latent_down, "attn_latent_down", rot, W, L.w_in, ldw, la.cr, rot, rotp, 0, 0, 0, rank + rot, rank));
    unsigned short *wq = nullptr, *wkv = nullptr;
    CH_TRY(alloc_matrix(c, H * (dimp + V), (size_t)la.ldl, &wkv));
    CH_TRY(pack_matrix(c, s.attn_key_up, "attn_key_up", H * s.attn_dim, rank, wkv, (size_t)la.ldl, 0, s.attn_dim, dimp));
    CH_TRY(pack_matrix(c, s.attn_value_up, "attn_value_up", H * s.attn_vdim, rank, wkv, (size_t)la.ldl, H * dimp, s.attn_vdim, V));
    CH_TRY(dalloc_n(c, H * rankp * dimp + 32, &wq));
    k_pack_transposed<<<dim3((unsigned)((rank + 255) / 256), (unsigned)s.attn_dim, (unsigned)H), 256, 0, dev->stream>>>((const unsigned short*)s.attn_key_up->ptr, (int)s.attn_dim,
                                                                                                             (int)rank, wq, la.rank, la.dim);
    CH_HIP(dev, hipGetLastError());
    la.w_q = wq;
    la.w_kv = wkv;
    CH_TRY(pack_matrix(c, s.attn_o, "attn_o", W, H * s.attn_vdim, L.w_o, (size_t)L.ldc, 0, W, W, 0, s.attn_vdim, V));
    float* p = nullptr;
    CH_TRY(pack_vector(c, s.attn_latent_norm, "attn_latent_norm", rank, &p, rank, rankp));
    la.norm = p;
    std::vector<double> f(rotp / 2 + 1, 0.0);
    for (size_t i = 0; i < rot / 2; i++) f[i] = pow(s.attn_rot_base, -2.0 * (double)i / (double)rot);
    double* df = nullptr;
    CH_TRY(dalloc_n(c, f.size(), &df));
    CH_HIP(dev, hipMemcpyAsync(df, f.data(), f.size() * sizeof(double), hipMemcpyHostToDevice, dev->stream));
    CH_HIP(dev, hipStreamSynchronize(dev->stream));  // f goes out of scope
    la.freq = df;
  }
  if (H && !rank) {
    if (!s.attn_q_norm != !s.attn_k_norm) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: attn_q_norm and attn_k_norm come together");
    float* np = nullptr;
    if (s.attn_q_norm) {
      CH_TRY(pack_vector(c, s.attn_q_norm, "attn_q_norm", H * s.attn_dim, &np, s.attn_dim, D));
      a.q_norm = np;
      CH_TRY(pack_vector(c, s.attn_k_norm, "attn_k_norm", G * s.attn_dim, &np, s.attn_dim, D));
      a.k_norm = np;
      a.q_mean = (int)(H * s.attn_dim);
      a.k_mean = (int)(G * s.attn_dim);
    }
    if (s.attn_vmix) {  // the first such layer's values are the ones the others take
      if (c->ld_vk && c->ld_vk != (int)(G * V)) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: layers that mix values must agree in their value heads");
      a.vmix = c->ld_vk ? VMIX_MIX : VMIX_KEEP;
      c->ld_vk = (int)(G * V);
      CH_TRY(pack_vector(c, s.attn_vmix, "attn_vmix", 1, &np));
      a.lambda = np;
    }
    CH_TRY(pack_matrix(c, s.attn_q, "attn_q", H * s.attn_dim, W, L.w_in, ldw, a.cq, s.attn_dim, D));
    CH_TRY(pack_matrix(c, s.attn_k, "attn_k", G * s.attn_dim, W, L.w_in, ldw, a.ck, s.attn_dim, D));
    CH_TRY(pack_matrix(c, s.attn_v, "attn_v", G * s.attn_vdim, W, L.w_in, ldw, a.cv, s.attn_vdim, V));
    if (a.gate == GATE_HEAD) CH_TRY(pack_matrix(c, s.attn_gate, "attn_gate", H, W, L.w_in, ldw, a.cg, H, H));
    if (a.gate == GATE_ELEMENT) CH_TRY(pack_matrix(c, s.attn_gate, "attn_gate", H * s.attn_vdim, W, L.w_in, ldw, a.cg, s.attn_vdim, V));
    CH_TRY(pack_matrix(c, s.attn_o, "attn_o", W, H * s.attn_vdim, L.w_o, (size_t)L.ldc, 0, W, W, 0, s.attn_vdim, V));
    if (!s.attn_bias_amp != !s.attn_bias_rate) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: attn_bias_amp and attn_bias_rate come together");
    float* p = nullptr;
    if (s.attn_bias_amp) {
      CH_TRY(pack_vector(c, s.attn_bias_amp, "attn_bias_amp", H, &p));
      a.amp = p;
      CH_TRY(pack_vector(c, s.attn_bias_rate, "attn_bias_rate", H, &p));
      a.rate = p;
    }
    if (s.attn_sink) {
      CH_TRY(pack_vector(c, s.attn_sink, "attn_sink", H, &p));
      a.sink = p;
    }
  }
  if (Hl) {
    CH_TRY(pack_matrix(c, s.lin_q, "lin_q", Hl * s.lin_dim, W, L.w_in, ldw, l.cq, s.lin_dim, Dl));
    CH_TRY(pack_matrix(c, s.lin_k, "lin_k", Hl * s.lin_dim, W, L.w_in, ldw, l.ck, s.lin_dim, Dl));
    CH_TRY(pack_matrix(c, s.lin_v, "lin_v", Hl * s.lin_vdim, W, L.w_in, ldw, l.cv, s.lin_vdim, Vl));
    CH_TRY(pack_matrix(c, s.lin_gate, "lin_gate", Hl * s.lin_vdim, W, L.w_in, ldw, l.cg, s.lin_vdim, Vl));
    CH_TRY(pack_matrix(c, s.lin_o, "lin_o", W, Hl * s.lin_vdim, L.w_o, (size_t)L.ldc, 0, W, W, L.lin_off, s.lin_vdim, Vl));
    float* p = nullptr;
    CH_TRY(pack_vector(c, s.lin_norm, "lin_norm", Hl * s.lin_vdim, &p, s.lin_vdim, Vl));
    l.norm = p;
    std::vector<float> pw(Hl * LIN_POW);
    for (size_t h = 0; h < Hl; h++)
      for (int n = 0; n < LIN_POW; n++) pw[h * LIN_POW + n] = (float)pow(s.lin_decay[h], (double)n);
    CH_TRY(dalloc_n(c, pw.size(), &p));
    CH_HIP(dev, hipMemcpyAsync(p, pw.data(), pw.size() * 4, hipMemcpyHostToDevice, dev->stream));
    CH_HIP(dev, hipStreamSynchronize(dev->stream));  // pw goes out of scope
    l.decay = p;
  }
  CH_TRY(pack_norm(c, s.norm1, "norm1", &L.norm1));
  if (c->streams) CH_TRY(pack_connection(c, s.hc1_in, s.hc1_out, s.hc1_mix, L.hc[0]));
  if (s.ff) {
    CH_TRY(pack_norm(c, s.norm2, "norm2", &L.norm2));
    if (c->streams) CH_TRY(pack_connection(c, s.hc2_in, s.hc2_out, s.hc2_mix, L.hc[1]));
    L.glu = s.ff_gate != nullptr;
    CH_TRY(alloc_matrix(c, s.ff * (L.glu ? 2 : 1), ldw, &L.w_up));
    CH_TRY(alloc_matrix(c, W, (size_t)L.ldu, &L.w_down));
    if (L.glu) {  // gate j, up j, gate j + 1, ..
      CH_TRY(pack_matrix(c, s.ff_gate, "ff_gate", s.ff, W, L.w_up, ldw, 0, 1, 2));
      CH_TRY(pack_matrix(c, s.ff_up, "ff_up", s.ff, W, L.w_up, ldw, 1, 1, 2));
    } else {
      CH_TRY(pack_matrix(c, s.ff_up, "ff_up", s.ff, W, L.w_up, ldw, 0, s.ff, s.ff));
    }
    CH_TRY(pack_matrix(c, s.ff_down, "ff_down", W, s.ff, L.w_down, (size_t)L.ldu, 0, W, W));
    if (L.glu) return 0;
    float* raw = nullptr;
    CH_TRY(pack_vector(c, s.ff_act, "ff_act", 2, &raw));
    CH_TRY(dalloc_n(c, 2, &L.xielu));
    k_xielu_consts<<<1, 1, 0, dev->stream>>>(raw, L.xielu);
    CH_HIP(dev, hipGetLastError());
  }
  return 0;
}

// ---- launches with the measurement hook's event pair ---------------------------------------------------------------------------------
struct Prof {
  crabml_hip_device* dev;
  crabml_hip_device::ProfRec r{};
  bool on;
  Prof(crabml_hip_device* d, bool enabled, int stage, double bytes) : dev(d), on(enabled && d->prof_on) {
    if (on) on = prof_begin(d, &r, CRABML_HIP_BF16, (uint32_t)stage, bytes) == 0;
  }
  ~Prof() {
    if (on) prof_end(dev, &r);
  }
  crabml_hip_device::ProfRec* rec() { return on ? &r : nullptr; }
};

// a decode linear: up to two rows on the vector kernel, more on the matrix cores
template <int IN, int OUT>
void step_linear(Ctx* c, crabml_hip_device::ProfRec* rec, const GemvBf16& g) {
  if (g.nb <= 2)
    launch_gemv_bf16<IN, OUT>(c->dev->stream, rec, g);
  else
    launch_gemv16_bf16<IN, OUT>(c->dev->stream, rec, g, c->f32);
}

MixStep mix_step(const Ctx* c, const Run& run, int B) {
  const Layer& L = c->layers[run.layer];
  MixStep m;
  m.at = L.at;
  m.li = L.li;
  m.rs = run.rs;
  m.seq = c->st_seq;
  m.proj = c->st_proj;
  m.cat = c->st_cat;
  m.ss = c->st_ss;
  m.part = c->st_part;
  m.tick = c->st_tick;
  m.v_kept = c->st_vk;
  m.ld_vk = c->ld_vk;
  m.B = B;
  m.ldp = L.n_in;
  m.ldc = L.ldc;
  m.lin_off = L.lin_off;
  m.splits = L.splits;
  m.head_blocks = L.head_blocks;
  return m;
}

// what is added to x behind the last linear of run r: what belongs in front of run r + 1
void next_adds(const Ctx* c, size_t r, const float* emb, const float** rows, const float** vec) {
  *rows = *vec = nullptr;
  if (r + 1 < c->runs.size()) {
    *rows = c->runs[r + 1].add_emb ? emb : nullptr;
    *vec = c->runs[r + 1].add_vec;
  }
}

// the residual streams behind sublayer q (0: mixer, 1: feed-forward) of run r, and the gain of the norm that reads them next
StreamMix streams_behind(const Ctx* c, size_t r, int q, size_t stride, const float** gain) {
  const Layer& L = c->layers[c->runs[r].layer];
  StreamMix m;
  m.n = c->streams;
  m.stride = stride;
  m.coef = L.hc[q].coef;
  if (q == 0 && L.ff) {
    m.in = L.hc[1].in;
    *gain = L.norm2;
  } else if (r + 1 < c->runs.size()) {
    const Layer& N = c->layers[c->runs[r + 1].layer];
    m.in = N.hc[0].in;
    *gain = N.norm1;
  } else {
    m.in = c->ones;
    *gain = c->final_norm;
  }
  return m;
}
// in front of the first layer
StreamMix streams_at_start(const Ctx* c, size_t stride) {
  StreamMix m;
  m.n = c->streams;
  m.stride = stride;
  m.in = c->streams ? c->layers[c->runs[0].layer].hc[0].in : nullptr;
  return m;
}
// an RMS norm and a linear behind it
template <int OUT>
void normed_linear(Ctx* c, crabml_hip_device::ProfRec* rec, const GemvBf16& g) {
  if (c->streams)
    step_linear<GEMV_IN_RMSV, OUT>(c, rec, g);
  else
    step_linear<GEMV_IN_RMS, OUT>(c, rec, g);
}

// the classifier on f32 rows
void head_rows(Ctx* c, const float* x, int B, bool prof) {
  GemvBf16 g;
  g.w = c->head;
  g.x = x;
  g.out = c->st_logits;
  g.N = g.ldo = c->vocab;
  g.K = g.ldw = g.ldx = c->ldx;
  g.nb = B;
  g.mean_n = c->width;
  g.eps = c->cfg.norm_eps;
  g.gain = c->final_norm;
  g.cap = c->cfg.logit_softcap;
  Prof p(c->dev, prof, ST_STEP + ST_HEAD, (double)c->vocab * c->ldx * 2);
  normed_linear<GEMV_OUT_SOFTCAP>(c, p.rec(), g);
}

template <typename T>
int latent_step(Ctx* c, const Run& run, int B, bool prof) {
  const Layer& L = c->layers[run.layer];
  LatStep m;
  m.at = L.at;
  m.la = L.la;
  m.rs = run.rs;
  m.seq = c->st_seq;
  m.proj = c->st_proj;
  m.q = c->st_q;
  m.part = c->st_lpart;
  m.cat = c->st_cat;
  m.B = B;
  m.ldp = L.n_in;
  m.ldc = L.ldc;
  m.splits = latent_splits(B, L.at.H);
  hipStream_t st = c->dev->stream;
  {
    Prof p(c->dev, prof, ST_STEP + ST_LAT, (double)L.at.H * L.la.rank * L.la.dim * 2);
    launch_latent_query<T>(st, p.rec(), m);
  }
  {
    Prof p(c->dev, prof, ST_STEP + ST_MIX, 0.0);
    CH_TRY(launch_latent_attn<T>(c->dev, p.rec(), m));
  }
  Prof p(c->dev, prof, ST_STEP + ST_ROWS, (double)L.at.H * L.la.rank * L.at.V * 2);
  launch_latent_value<T>(st, p.rec(), m);
  return 0;
}


int enqueue_step(Ctx* c, int B, bool sample, bool prof) {
  crabml_hip_device* dev = c->dev;
  hipStream_t st = dev->stream;
  const float eps = c->cfg.norm_eps;
  const size_t stride = (size_t)HYB_STEP_ROWS * c->ldx;
  const float* next_gain = nullptr;
  float* x_in = c->streams ? c->st_in : c->st_x;  // what a norm reads
  k_embed_step<<<dim3((c->width + 255) / 256, B), 256, 0, st>>>(c->embed, c->st_seq, c->width, c->ldx, c->cfg.embed_scale, c->freq, c->st_x,
                                                               c->keep_emb ? c->st_emb : nullptr, c->runs[0].add_vec, streams_at_start(c, stride), c->st_in);
  for (size_t r = 0; r < c->runs.size(); r++) {
    const Run& run = c->runs[r];
    const Layer& L = c->layers[run.layer];
    const float *add_rows, *add_vec;
    next_adds(c, r, c->st_emb, &add_rows, &add_vec);
    {
      GemvBf16 g;
      g.w = L.w_in;
      g.x = x_in;
      g.out = c->st_proj;
      g.N = g.ldo = L.n_in;
      g.K = g.ldw = g.ldx = c->ldx;
      g.nb = B;
      g.mean_n = c->width;
      g.eps = eps;
      g.gain = L.norm1;
      g.act = L.act;
      g.bias = L.bias_in;
      Prof p(dev, prof, ST_STEP + ST_IN, (double)L.n_in * c->ldx * 2);
      normed_linear<GEMV_OUT_ACT>(c, p.rec(), g);
    }
    if (L.la.rank) {
      CH_TRY(c->f32 ? latent_step<float>(c, run, B, prof) : latent_step<unsigned short>(c, run, B, prof));
    } else {
      const MixStep m = mix_step(c, run, B);
      Prof p(dev, prof, ST_STEP + ST_MIX, 0.0);
      if (c->f32)
        launch_mix_step<float>(st, p.rec(), m);
      else
        launch_mix_step<unsigned short>(st, p.rec(), m);
    }
    {
      GemvBf16 g;
      g.w = L.w_o;
      g.x = c->st_cat;
      g.out = c->st_x;
      g.N = c->width;
      g.ldo = g.ld_add = c->ldx;
      g.K = g.ldw = g.ldx = L.ldc;
      g.nb = B;
      g.mean_n = L.li.H ? L.li.H * L.li.v_true : 1;
      g.eps = eps;
      g.k_split = L.lin_off;
      g.n_ss = L.li.H * L.li.slices;
      g.ss = c->st_ss;
      if (!L.ff) {
        g.add_rows = add_rows;
        g.add_vec = add_vec;
      }
      Prof p(dev, prof, ST_STEP + ST_OUT, (double)c->width * L.ldc * 2);
      if (c->streams) {
        g.bias = L.bias_o;
        g.sm = streams_behind(c, r, 0, stride, &next_gain);
        g.u = c->st_in;
        step_linear<GEMV_IN_SPLIT, GEMV_OUT_STREAMS>(c, p.rec(), g);
      } else {
        step_linear<GEMV_IN_SPLIT, GEMV_OUT_RESIDUAL>(c, p.rec(), g);
      }
    }
    if (!L.ff) continue;
    {
      GemvBf16 g;
      g.w = L.w_up;
      g.x = x_in;
      g.out = c->st_u;
      g.N = L.glu ? 2 * L.ff : L.ff;
      g.ldo = L.ldu;
      g.K = g.ldw = g.ldx = c->ldx;
      g.nb = B;
      g.mean_n = c->width;
      g.eps = eps;
      g.gain = L.norm2;
      g.xielu = L.xielu;
      Prof p(dev, prof, ST_STEP + ST_UP, (double)g.N * c->ldx * 2);
      if (L.glu)
        normed_linear<GEMV_OUT_GLU>(c, p.rec(), g);
      else
        normed_linear<GEMV_OUT_XIELU>(c, p.rec(), g);
    }
    {
      GemvBf16 g;
      g.w = L.w_down;
      g.x = c->st_u;
      g.out = c->st_x;
      g.N = c->width;
      g.ldo = g.ld_add = c->ldx;
      g.K = g.ldw = g.ldx = L.ldu;
      g.nb = B;
      g.add_rows = add_rows;
      g.add_vec = add_vec;
      Prof p(dev, prof, ST_STEP + ST_DOWN, (double)c->width * L.ldu * 2);
      if (c->streams) {
        g.sm = streams_behind(c, r, 1, stride, &next_gain);
        g.u = c->st_in;
        step_linear<GEMV_IN_PLAIN, GEMV_OUT_STREAMS>(c, p.rec(), g);
      } else {
        step_linear<GEMV_IN_PLAIN, GEMV_OUT_RESIDUAL>(c, p.rec(), g);
      }
    }
  }
  head_rows(c, x_in, B, prof);
  if (sample) {
    k_argmax_partial<<<dim3(ARGMAX_BLOCKS, B), 256, 0, st>>>(c->st_logits, c->vocab, c->am_val, c->am_idx, 0, c->vocab);
    k_argmax_rows_step<<<B, 64, 0, st>>>(c->am_val, c->am_idx, ARGMAX_BLOCKS, c->st_seq, c->st_count, c->st_out, (int)c->st_out_cap);
    k_step_advance<<<1, 1, 0, st>>>(c->st_count);
  }
  CH_HIP(dev, hipGetLastError());
  return 0;
}

// one decode step of B rows from its graph (captured when that batch size first comes up), or eagerly
int run_step(Ctx* c, int B, bool sample) {
  crabml_hip_device* dev = c->dev;
  if ((c->cfg.flags & CRABML_HIP_HYBRID_NO_GRAPH) || dev->prof_on) return enqueue_step(c, B, sample, true);
  auto& slot = c->graphs[B * 2 + (sample ? 1 : 0)];
  if (!slot.second) {
    CH_HIP(dev, hipStreamBeginCapture(dev->stream, hipStreamCaptureModeThreadLocal));
    const int rc = enqueue_step(c, B, sample, false);
    hipGraph_t graph = nullptr;
    const hipError_t e = hipStreamEndCapture(dev->stream, &graph);
    hipGraphExec_t exec = nullptr;
    if (rc != 0 || e != hipSuccess || !graph || hipGraphInstantiate(&exec, graph, nullptr, nullptr, 0) != hipSuccess) {
      if (graph) (void)hipGraphDestroy(graph);
      (void)hipGetLastError();
      CH_BAIL(dev, CRABML_HIP_UNEXPECTED, "hybrid: hipGraph capture / instantiate of the decode step failed");
    }
    slot = {graph, exec};
  }
  CH_HIP(dev, hipGraphLaunch(slot.second, dev->stream));
  return 0;
}

int step_begin(Ctx* c, size_t n, const size_t* seqs, const uint32_t* tokens) {
  crabml_hip_device* dev = c->dev;
  if (c->h_seq_next == META_SLOTS) {  // every slot may still be waiting for its copy
    CH_HIP(dev, hipStreamSynchronize(dev->stream));
    c->h_seq_next = 0;
  }
  StepSeq* h = c->h_seq + (size_t)HYB_STEP_ROWS * c->h_seq_next++;
  for (size_t i = 0; i < n; i++) {
    h[i].token = (int)tokens[i];
    h[i].pos = (int)c->seqs[seqs[i]].len;
    h[i].slab = c->seqs[seqs[i]].slab;
  }
  CH_HIP(dev, hipMemcpyAsync(c->st_seq, h, n * sizeof(StepSeq), hipMemcpyHostToDevice, dev->stream));
  return 0;
}

// ---- prompt pass -------------------------------------------------------------------------------------------------------------------
int pass_alloc(Ctx* c) {
  if (c->rows_cap) return 0;
  crabml_hip_device* dev = c->dev;
  const size_t R = align_up(c->cfg.pass_rows ? c->cfg.pass_rows : 2048, 256), P = (size_t)c->planes;
  size_t lin = 0;
  for (const Layer& L : c->layers) lin = std::max(lin, (size_t)L.li.H * L.li.V);
  const size_t S = c->streams ? (size_t)c->streams : 1, e = c->f32 ? 4 : 2, Hc = c->hist ? align_up(std::max(R, c->hist), 256) : 0;
  CH_TRY(dalloc_n(c, S * R * c->ldx, &c->pf_x));
  if (c->keep_emb) CH_TRY(dalloc_n(c, R * c->ldx, &c->pf_emb));
  CH_TRY(dalloc_n(c, P * R * c->ldx, &c->pf_xp));
  CH_TRY(dalloc(c, R * c->ld_proj * e, &c->pf_proj));
  if (c->ld_vk) CH_TRY(dalloc(c, R * c->ld_vk * e, &c->pf_vk));
  if (c->ld_kv) {
    CH_TRY(dalloc_n(c, P * (R + Hc) * c->ld_lat, &c->pf_lat));
    CH_TRY(dalloc(c, (R + Hc) * c->ld_rot * e, &c->pf_rot));
    CH_TRY(dalloc(c, (R + Hc) * c->ld_kv * e, &c->pf_kv));
  }
  CH_TRY(dalloc_n(c, P * R * c->ld_cat, &c->pf_cat));
  CH_TRY(dalloc_n(c, R * lin, &c->pf_lin));
  CH_TRY(dalloc_n(c, P * R * c->ld_u, &c->pf_u));
  CH_TRY(dalloc_n(c, R * c->n_sq, &c->pf_sq));
  c->pf_scratch.floats = (size_t)16 << 20;
  CH_TRY(dalloc(c, c->pf_scratch.floats * sizeof(float), (void**)&c->pf_scratch.partials, false));
  CH_TRY(dalloc_n(c, GEMM_TICKS, &c->pf_scratch.ticks));
  CH_TRY(dalloc_n(c, P * LOGIT_ROWS * c->ldx, &c->pf_gp));
  CH_TRY(dalloc_n(c, LOGIT_ROWS * c->n_sq, &c->pf_gsq));
  CH_TRY(dalloc_n(c, LOGIT_ROWS * c->vocab, &c->pf_logits));
  // seqs | tiles, small and big (a tile is at least one row) | rows, earlier positions behind them | tokens | wanted rows
  c->meta_bytes = R * (sizeof(PassSeq) + 2 * sizeof(PassTile) + 2 * sizeof(int)) + (R + Hc) * sizeof(PassRow);
  CH_TRY(dalloc(c, c->meta_bytes, (void**)&c->meta));
  CH_HIP(dev, hipHostMalloc((void**)&c->h_meta, c->meta_bytes * META_SLOTS, hipHostMallocDefault));
  CH_HIP(dev, hipStreamCreateWithFlags(&c->side, hipStreamNonBlocking));
  CH_HIP(dev, hipEventCreateWithFlags(&c->fork, hipEventDisableTiming));
  CH_HIP(dev, hipEventCreateWithFlags(&c->join, hipEventDisableTiming));
  c->rows_cap = R;
  c->hist_cap = Hc;
  return 0;
}

struct PassTiles {  // query tiles of 64 and of 128 rows
  const PassTile* list[2];
  size_t n[2];
};
struct Part {  // rows of one sequence in one pass
  size_t seq, n;
  const uint32_t* tokens;
  std::vector<int> want;  // places among these rows
};

template <typename T, int KC, int VC, bool LAT>
void launch_attn_cls(Ctx* c, crabml_hip_device::ProfRec* rec, MixRows<T> m, const PassTiles& tiles) {
  constexpr int big = AttnTile<T, KC, VC>::RT - 1;
  m.tiles = tiles.list[big];
  m.n_tiles = (int)tiles.n[big];
  launch_k(c->dev->stream, rec, k_attn_rows<T, KC, VC, sizeof(T) == 2 ? 1 : 3, LAT>, dim3(m.n_tiles, m.at.H), dim3(256), 0, m);
}
template <typename T, bool LAT>
void launch_attn(Ctx* c, const MixRows<T>& m, const PassTiles& tiles) {
  Prof p(c->dev, true, ST_PASS + ST_MIX, 0.0);
  const int w = std::max(m.at.D, m.at.V);
  if (w <= 64) return launch_attn_cls<T, 64, 64, LAT>(c, p.rec(), m, tiles);
  if (w <= 128) return launch_attn_cls<T, 128, 128, LAT>(c, p.rec(), m, tiles);
  if constexpr (LAT && sizeof(T) == 2)
    if (w <= 192 && m.at.V <= 128) return launch_attn_cls<T, 192, 128, LAT>(c, p.rec(), m, tiles);
  launch_attn_cls<T, 256, 256, LAT>(c, p.rec(), m, tiles);
}
template <typename T, int CLS>
int launch_linear_cls(Ctx* c, hipStream_t st, crabml_hip_device::ProfRec* rec, const MixRows<T>& m, size_t n_seq) {
  const size_t lds = LinTile<T, CLS>::LDS;
  CH_HIP(c->dev, raise_dyn_lds(c->dev, (const void*)k_linear_rows<T, CLS>, (int)lds));
  launch_k(st, rec, k_linear_rows<T, CLS>, dim3(m.li.H * m.li.slices, (unsigned)n_seq), dim3(256), lds, m);
  return 0;
}

template <typename T>
int mix_rows(Ctx* c, const Run& run, const PassSeq* seqs, size_t n_seq, const PassTiles& tiles, const PassRow* rows, size_t n_rows, size_t n_hist) {
  constexpr int P = sizeof(T) == 2 ? 1 : 3;
  const Layer& L = c->layers[run.layer];
  MixRows<T> m;
  m.at = L.at;
  m.li = L.li;
  m.rs = run.rs;
  m.seqs = seqs;
  m.rows = rows;
  m.la = L.la;
  m.M = (int)n_rows;
  m.v_kept = (T*)c->pf_vk;
  m.ld_vk = c->ld_vk;
  m.proj = (const T*)c->pf_proj;
  m.cat = c->pf_cat;
  m.cat_plane = c->rows_cap * (size_t)c->ld_cat;
  m.lin = c->pf_lin;
  m.ldp = L.n_in;
  m.ldc = L.ldc;
  m.lin_off = L.lin_off;
  if (L.la.rank) {
    const int all = (int)(n_rows + n_hist);
    m.lat = c->pf_lat;
    m.lat_plane = (c->rows_cap + c->hist_cap) * (size_t)c->ld_lat;
    m.rot = (T*)c->pf_rot;
    m.kv = (const T*)c->pf_kv;
    {
      Prof p(c->dev, true, ST_PASS + ST_ROWS, 0.0);
      launch_k(c->dev->stream, p.rec(), k_latent_rows<T, P>, dim3(all), dim3(256), 0, m);
    }
    {
      GemmBf16 g;
      g.a = c->pf_lat;
      g.a_plane = m.lat_plane;
      g.w = L.la.w_kv;
      g.M = all;
      g.N = g.ldo = L.at.H * (L.la.dim + L.at.V);
      g.K = L.la.ldl;
      g.out = c->pf_kv;
      Prof p(c->dev, true, ST_PASS + ST_LAT, 0.0);
      launch_gemm_bf16(c->dev, p.rec(), P, sizeof(T) == 4 ? GEMM_OUT_ACT_F32 : GEMM_OUT_ACT_BF16, g, c->pf_scratch);
    }
    launch_attn<T, true>(c, m, tiles);
    Prof p(c->dev, true, ST_PASS + ST_ROWS, 0.0);
    launch_k(c->dev->stream, p.rec(), k_latent_append<T, P>, dim3((unsigned)n_rows), dim3(256), 0, m);
    return 0;
  }
  if (L.at.H && (L.at.q_norm || L.at.vmix)) {
    Prof p(c->dev, true, ST_PASS + ST_ROWS, 0.0);
    launch_k(c->dev->stream, p.rec(), k_qkv_rows<T>, dim3((unsigned)n_rows), dim3(256), 0, m);
  }
  // the linear branch is a chain of blocks on few CUs: beside the softmax branch, when both are long enough to hide a fork
  hipStream_t st = c->dev->stream, lin_st = st;
  if (L.at.H && L.li.H && n_rows >= 192 && !c->dev->prof_on) {
    lin_st = c->side;
    CH_HIP(c->dev, hipEventRecord(c->fork, st));
    CH_HIP(c->dev, hipStreamWaitEvent(lin_st, c->fork, 0));
  }
  if (L.li.H) {
    Prof p(c->dev, true, ST_PASS + ST_LIN, 0.0);
    if (L.li.D <= 64)
      CH_TRY((launch_linear_cls<T, 64>(c, lin_st, p.rec(), m, n_seq)));
    else if (L.li.D <= 128)
      CH_TRY((launch_linear_cls<T, 128>(c, lin_st, p.rec(), m, n_seq)));
    else
      CH_TRY((launch_linear_cls<T, 256>(c, lin_st, p.rec(), m, n_seq)));
  }
  if (lin_st != st) CH_HIP(c->dev, hipEventRecord(c->join, lin_st));
  if (L.at.H) launch_attn<T, false>(c, m, tiles);
  if (lin_st != st) CH_HIP(c->dev, hipStreamWaitEvent(st, c->join, 0));
  Prof p(c->dev, true, ST_PASS + ST_ROWS, 0.0);
  launch_k(c->dev->stream, p.rec(), k_mix_rows<T, P>, dim3((unsigned)n_rows), dim3(256), 0, m, c->cfg.norm_eps);
  return 0;
}

// one pass over the rows of `parts`; logits of the wanted rows go to *logits, which advances
int run_pass(Ctx* c, const std::vector<Part>& parts, float** logits) {
  crabml_hip_device* dev = c->dev;
  hipStream_t st = dev->stream;
  CH_TRY(pass_alloc(c));
  if (c->h_meta_next == META_SLOTS) {
    CH_HIP(dev, hipStreamSynchronize(st));
    c->h_meta_next = 0;
  }
  const size_t R = c->rows_cap;
  char* hm = c->h_meta + c->meta_bytes * c->h_meta_next++;
  const size_t o_tile = R * sizeof(PassSeq), o_row = o_tile + 2 * R * sizeof(PassTile), o_tok = o_row + (R + c->hist_cap) * sizeof(PassRow), o_want = o_tok + R * sizeof(int);
  PassSeq* hs = (PassSeq*)hm;
  PassTile* ht[2] = {(PassTile*)(hm + o_tile), (PassTile*)(hm + o_tile) + R};
  PassRow* hr = (PassRow*)(hm + o_row);
  int *hk = (int*)(hm + o_tok), *hw = (int*)(hm + o_want);
  size_t n_tiles[2] = {0, 0}, M = 0, nw = 0;
  for (size_t i = 0; i < parts.size(); i++) {
    const Part& p = parts[i];
    const Seq& s = c->seqs[p.seq];
    hs[i] = PassSeq{(int)M, (int)p.n, (int)s.len, (int)M, s.slab};
    for (size_t b = 0; b < 2; b++)
      for (size_t r = 0; r < p.n; r += 64 << b)
        ht[b][n_tiles[b]++] = PassTile{(int)i, (int)(M + r), (int)(s.len + r), (int)std::min<size_t>(64 << b, p.n - r)};
    for (int w : p.want) hw[nw++] = (int)M + w;
    for (size_t r = 0; r < p.n; r++) {
      hr[M + r] = PassRow{(int)i, (int)(s.len + r)};
      hk[M + r] = (int)p.tokens[r];
    }
    M += p.n;
  }
  size_t n_hist = 0;  // earlier positions that latent layers read again
  for (size_t i = 0; i < parts.size(); i++) {
    const int len = (int)c->seqs[parts[i].seq].len, n = (int)std::min(c->hist, (size_t)len);
    for (int p = len - n; p < len; p++) hr[M + n_hist++] = PassRow{(int)i, p};
    hs[i].hist_end = (int)(M + n_hist);
  }
  CH_HIP(dev, hipMemcpyAsync(c->meta, hm, c->meta_bytes, hipMemcpyHostToDevice, st));
  const PassSeq* ds = (const PassSeq*)c->meta;
  const PassTiles dt = {{(const PassTile*)(c->meta + o_tile), (const PassTile*)(c->meta + o_tile) + R}, {n_tiles[0], n_tiles[1]}};
  const PassRow* dr = (const PassRow*)(c->meta + o_row);
  const int *dk = (const int*)(c->meta + o_tok), *dw = (const int*)(c->meta + o_want);
  const size_t xp = R * (size_t)c->ldx;
  const float eps = c->cfg.norm_eps;
  float* emb = c->keep_emb ? c->pf_emb : nullptr;
  const size_t stride = R * (size_t)c->ldx;
  const float* next_gain = c->streams ? c->layers[c->runs[0].layer].norm1 : nullptr;
  {
    const StreamMix sm = streams_at_start(c, stride);
    auto embed = c->f32 ? k_embed_rows<3> : k_embed_rows<1>;
    embed<<<(unsigned)M, 256, 0, st>>>(c->embed, dk, dr, c->width, c->ldx, c->cfg.embed_scale, c->freq, c->pf_x, emb, c->runs[0].add_vec, c->pf_xp, xp, c->pf_sq, c->n_sq, sm,
                                       next_gain);
  }
  auto normed = [&](const unsigned short* w, int n, const float* gain) {
    GemmBf16 g;
    g.a = c->pf_xp;
    g.a_plane = xp;
    g.w = w;
    g.M = (int)M;
    g.N = n;
    g.K = c->ldx;
    g.sq_in = c->pf_sq;
    g.n_sq = c->n_sq;
    g.mean_n = c->width;
    g.eps = eps;
    g.gain = c->streams ? nullptr : gain;  // (a gain per element is in the planes)
    return g;
  };
  auto residual = [&](const unsigned short* a, size_t a_plane, const unsigned short* w, int k) {
    GemmBf16 g;
    g.a = a;
    g.a_plane = a_plane;
    g.w = w;
    g.M = (int)M;
    g.N = c->width;
    g.K = k;
    g.x = c->pf_x;
    g.ldx = c->ldx;
    g.planes = c->pf_xp;
    g.p_plane = xp;
    g.ldp = c->ldx;
    g.sq_out = c->pf_sq;
    g.n_sq_out = c->n_sq;
    return g;
  };
  for (size_t r = 0; r < c->runs.size(); r++) {
    const Run& run = c->runs[r];
    const Layer& L = c->layers[run.layer];
    const float *add_rows, *add_vec;
    next_adds(c, r, c->pf_emb, &add_rows, &add_vec);
    {
      GemmBf16 g = normed(L.w_in, L.n_in, L.norm1);
      g.out = c->pf_proj;
      g.ldo = L.n_in;
      g.act = L.act;
      g.bias = L.bias_in;
      Prof p(dev, true, ST_PASS + ST_IN, 0.0);
      launch_gemm_bf16(dev, p.rec(), c->planes, c->f32 ? GEMM_OUT_ACT_F32 : GEMM_OUT_ACT_BF16, g, c->pf_scratch);
    }
    if (c->f32)
      CH_TRY(mix_rows<float>(c, run, ds, parts.size(), dt, dr, M, n_hist));
    else
      CH_TRY(mix_rows<unsigned short>(c, run, ds, parts.size(), dt, dr, M, n_hist));
    {
      GemmBf16 g = residual(c->pf_cat, R * (size_t)c->ld_cat, L.w_o, L.ldc);
      if (!L.ff) {
        g.add_rows = add_rows;
        g.add_vec = add_vec;
      }
      if (c->streams) {
        g.bias = L.bias_o;
        g.sm = streams_behind(c, r, 0, stride, &g.gain_next);
      }
      Prof p(dev, true, ST_PASS + ST_OUT, 0.0);
      launch_gemm_bf16(dev, p.rec(), c->planes, c->streams ? GEMM_OUT_STREAMS : GEMM_OUT_RESIDUAL, g, c->pf_scratch);
    }
    if (!L.ff) continue;
    {
      GemmBf16 g = normed(L.w_up, L.glu ? 2 * L.ff : L.ff, L.norm2);
      g.planes = c->pf_u;
      g.p_plane = R * (size_t)c->ld_u;
      g.ldp = L.ldu;
      g.xielu = L.xielu;
      Prof p(dev, true, ST_PASS + ST_UP, 0.0);
      launch_gemm_bf16(dev, p.rec(), c->planes, L.glu ? GEMM_OUT_GLU : GEMM_OUT_XIELU, g, c->pf_scratch);
    }
    {
      GemmBf16 g = residual(c->pf_u, R * (size_t)c->ld_u, L.w_down, L.ldu);
      g.add_rows = add_rows;
      g.add_vec = add_vec;
      if (c->streams) g.sm = streams_behind(c, r, 1, stride, &g.gain_next);
      Prof p(dev, true, ST_PASS + ST_DOWN, 0.0);
      launch_gemm_bf16(dev, p.rec(), c->planes, c->streams ? GEMM_OUT_STREAMS : GEMM_OUT_RESIDUAL, g, c->pf_scratch);
    }
  }
  for (size_t w0 = 0; w0 < nw; w0 += LOGIT_ROWS) {
    const size_t n = std::min(LOGIT_ROWS, nw - w0);
    const float* src = c->pf_logits;
    StreamMix sum = streams_at_start(c, stride);
    if (c->streams) sum.in = c->ones;
    if (n <= 8) {  // the decode step's classifier
      float* x = c->streams ? c->st_in : c->st_x;
      k_gather_rows<0><<<(unsigned)n, 256, 0, st>>>(c->pf_x, c->ldx, c->width, dw + w0, x, nullptr, 0, nullptr, 0, sum, nullptr);
      head_rows(c, x, (int)n, true);
      src = c->st_logits;
    } else {
      const size_t gp = LOGIT_ROWS * (size_t)c->ldx;
      auto gather = c->f32 ? k_gather_rows<3> : k_gather_rows<1>;
      gather<<<(unsigned)n, 256, 0, st>>>(c->pf_x, c->ldx, c->width, dw + w0, nullptr, c->pf_gp, gp, c->pf_gsq, c->n_sq, sum, c->streams ? c->final_norm : nullptr);
      GemmBf16 g = normed(c->head, c->vocab, c->final_norm);
      g.a = c->pf_gp;
      g.a_plane = gp;
      g.sq_in = c->pf_gsq;
      g.M = (int)n;
      g.out = c->pf_logits;
      g.ldo = c->vocab;
      g.cap = c->cfg.logit_softcap;
      Prof p(dev, true, ST_PASS + ST_HEAD, 0.0);
      launch_gemm_bf16(dev, p.rec(), c->planes, GEMM_OUT_SOFTCAP, g, c->pf_scratch);
    }
    CH_HIP(dev, hipMemcpyAsync(*logits, src, n * c->vocab * sizeof(float), hipMemcpyDeviceToHost, st));
    CH_HIP(dev, hipStreamSynchronize(st));
    *logits += n * c->vocab;
  }
  CH_HIP(dev, hipGetLastError());
  for (const Part& p : parts) c->seqs[p.seq].len += p.n;
  return 0;
}

int check_seq(const Ctx* c, size_t seq) {
  if (seq >= c->seqs.size() || !c->seqs[seq].open) CH_BAIL(c->dev, CRABML_HIP_BAD_INPUT, "hybrid: sequence %zu is not open", seq);
  return 0;
}

int create_impl(Ctx* c, const crabml_hip_hybrid_layer_t* layers, const crabml_hip_hybrid_weights_t& w) {
  crabml_hip_device* dev = c->dev;
  const auto& g = c->cfg;
  const size_t W = g.width;
  c->f32 = g.compute == CRABML_HIP_F32;
  c->planes = c->f32 ? 3 : 1;
  c->width = (int)W;
  c->vocab = (int)g.vocab_size;
  c->ldx = up(W, 64);
  c->n_sq = c->ldx / 64;
  c->keep_emb = g.loop_times > 1;
  c->streams = g.streams ? (int)g.streams : (g.flags & CRABML_HIP_HYBRID_NORM_VECTOR ? 1 : 0);
  CH_TRY(dalloc_n(c, HC_MAX, &c->ones));
  const std::vector<float> ones(HC_MAX, 1.f);
  CH_HIP(dev, hipMemcpyAsync(c->ones, ones.data(), HC_MAX * sizeof(float), hipMemcpyHostToDevice, dev->stream));
  CH_HIP(dev, hipStreamSynchronize(dev->stream));
  CH_TRY(alloc_matrix(c, g.vocab_size, (size_t)c->ldx, &c->head));
  CH_TRY(dalloc_n(c, g.vocab_size * W, &c->embed));
  CH_TRY(pack_matrix(c, w.embed, "embed", g.vocab_size, W, c->embed, W, 0, g.vocab_size, g.vocab_size));
  CH_TRY(pack_matrix(c, w.head ? w.head : w.embed, "head", g.vocab_size, W, c->head, (size_t)c->ldx, 0, g.vocab_size, g.vocab_size));
  CH_TRY(pack_norm(c, w.final_norm, "final_norm", &c->final_norm));
  if (g.loop_times) CH_TRY(pack_vector(c, w.loop_step, "loop_step", g.loop_times * W, &c->loop_step));
  c->layers.resize(g.n_layers);
  size_t part = 0, tick = 0, ss = 0, lat_q = 0, lat_part = 0;
  for (size_t i = 0; i < g.n_layers; i++) {
    Layer& L = c->layers[i];
    CH_TRY(build_layer(c, layers[i], L));
    c->ld_proj = std::max(c->ld_proj, L.n_in);
    c->ld_cat = std::max(c->ld_cat, L.ldc);
    c->ld_u = std::max(c->ld_u, L.ldu);
    if (L.la.rank) {
      const size_t row = (size_t)L.la.rank + L.la.rot;
      lat_q = std::max(lat_q, (size_t)HYB_STEP_ROWS * L.at.H * row);
      lat_part = std::max(lat_part, (size_t)HYB_STEP_ROWS * L.at.H * LAT_SPLITS * (L.la.rank + 2));
      c->ld_kv = std::max(c->ld_kv, L.at.H * (L.la.dim + L.at.V));
      c->ld_lat = std::max(c->ld_lat, L.la.ldl);
      c->ld_rot = std::max(c->ld_rot, L.la.rot);
      c->hist = std::max(c->hist, (size_t)L.at.rows - (L.at.window ? 1 : 0));
    } else if (L.at.H) {
      const size_t slots = (size_t)HYB_STEP_ROWS * L.at.G * L.head_blocks;
      part = std::max(part, slots * L.splits * mix_part_floats(L.at.V));
      tick = std::max(tick, slots);
    }
    ss = std::max(ss, (size_t)HYB_STEP_ROWS * L.li.H * L.li.slices);
  }
  // the order of layer runs, and each run's place in a sequence's slab
  auto add_run = [&](size_t layer, bool first, size_t t) {
    Run r;
    r.layer = (int)layer;
    const Layer& L = c->layers[layer];
    const size_t e = c->f32 ? 4 : 2;
    auto take = [&](size_t bytes) {
      const size_t at = c->slab_bytes;
      c->slab_bytes += align_up(bytes, 256);
      return at;
    };
    if (L.la.rank) {
      r.rs.k = take((size_t)L.at.rows * (L.la.rank + L.la.rot) * e);
    } else if (L.at.H) {
      r.rs.k = take((size_t)L.at.G * L.at.rows * L.at.D * e);
      r.rs.v = take((size_t)L.at.G * L.at.rows * L.at.V * e);
    }
    if (L.li.H) r.rs.s = take((size_t)L.li.H * L.li.D * L.li.V * 4);
    if (first) {
      r.add_emb = t > 0;
      r.add_vec = c->loop_step + t * W;
    }
    c->runs.push_back(r);
  };
  const size_t lo = g.loop_times ? g.loop_start : g.n_layers, hi = g.loop_times ? g.loop_stop : g.n_layers;
  for (size_t i = 0; i < lo; i++) add_run(i, false, 0);
  for (size_t t = 0; t < g.loop_times; t++)
    for (size_t i = lo; i < hi; i++) add_run(i, i == lo, t);
  for (size_t i = hi; i < g.n_layers; i++) add_run(i, false, 0);
  if (g.position_base > 0) {
    std::vector<double> f((W + 1) / 2);
    for (size_t i = 0; i < f.size(); i++) f[i] = pow(g.position_base, -2.0 * (double)i / (double)W);
    CH_TRY(dalloc_n(c, f.size(), &c->freq));
    CH_HIP(dev, hipMemcpyAsync(c->freq, f.data(), f.size() * sizeof(double), hipMemcpyHostToDevice, dev->stream));
    CH_HIP(dev, hipStreamSynchronize(dev->stream));
  }
  const size_t B = HYB_STEP_ROWS;
  CH_TRY(dalloc_n(c, B, &c->st_seq));
  CH_TRY(dalloc_n(c, 1, &c->st_count));
  CH_TRY(dalloc_n(c, (c->streams ? c->streams : 1) * B * c->ldx, &c->st_x));
  if (c->streams) CH_TRY(dalloc_n(c, B * c->ldx, &c->st_in));
  if (c->ld_vk) CH_TRY(dalloc_n(c, B * c->ld_vk, &c->st_vk));
  CH_TRY(dalloc_n(c, lat_q, &c->st_q));
  CH_TRY(dalloc_n(c, lat_part, &c->st_lpart));
  CH_TRY(dalloc_n(c, B * c->ldx, &c->st_emb));
  CH_TRY(dalloc_n(c, B * c->ld_proj, &c->st_proj));
  CH_TRY(dalloc_n(c, B * c->ld_cat, &c->st_cat));
  CH_TRY(dalloc_n(c, B * c->ld_u, &c->st_u));
  CH_TRY(dalloc_n(c, ss, &c->st_ss));
  CH_TRY(dalloc_n(c, part, &c->st_part));
  CH_TRY(dalloc_n(c, tick, &c->st_tick));
  CH_TRY(dalloc_n(c, B * c->vocab, &c->st_logits));
  c->st_out_cap = B * g.seq_len;
  CH_TRY(dalloc_n(c, c->st_out_cap, &c->st_out));
  CH_TRY(dalloc_n(c, B * ARGMAX_BLOCKS, &c->am_val));
  CH_TRY(dalloc_n(c, B * ARGMAX_BLOCKS, &c->am_idx));
  CH_HIP(dev, hipHostMalloc((void**)&c->h_seq, META_SLOTS * B * sizeof(StepSeq), hipHostMallocDefault));
  CH_HIP(dev, hipStreamSynchronize(dev->stream));
  return 0;
}

}  // namespace

extern "C" {

int crabml_hip_hybrid_create(crabml_hip_device_t* dev, const crabml_hip_hybrid_config_t* cfg, const crabml_hip_hybrid_layer_t* layers,
                             const crabml_hip_hybrid_weights_t* w, crabml_hip_hybrid_t** out) {
  if (!dev || !cfg || !layers || !w || !out) return CRABML_HIP_BAD_INPUT;
  *out = nullptr;
  CH_LIVE(dev);
  CH_USE(dev);
  CH_FLUSH(dev);
  if (!cfg->width || !cfg->vocab_size || !cfg->n_layers || !cfg->seq_len || cfg->width > 65536 || cfg->vocab_size > (1u << 24) || cfg->seq_len > (1u << 24))
    CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: width %zu, vocab %zu, %zu layers, %zu positions", cfg->width, cfg->vocab_size, cfg->n_layers, cfg->seq_len);
  if (cfg->compute != CRABML_HIP_BF16 && cfg->compute != CRABML_HIP_F32) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: compute is BF16 or F32, not %u", cfg->compute);
  if (cfg->loop_times && (cfg->loop_start >= cfg->loop_stop || cfg->loop_stop > cfg->n_layers))
    CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: loop over layers [%zu, %zu) of %zu", cfg->loop_start, cfg->loop_stop, cfg->n_layers);
  if (cfg->streams > HC_MAX) CH_BAIL(dev, CRABML_HIP_NOT_IMPLEMENTED, "hybrid: %zu residual streams (at most %d)", cfg->streams, HC_MAX);
  if (cfg->loop_times && (cfg->streams || (cfg->flags & CRABML_HIP_HYBRID_NORM_VECTOR)))
    CH_BAIL(dev, CRABML_HIP_NOT_IMPLEMENTED, "hybrid: a loop goes with a single residual row and norms of a single gain");
  Ctx* c = new Ctx();
  c->dev = dev;
  c->cfg = *cfg;
  const int rc = create_impl(c, layers, *w);
  if (rc != 0) {
    crabml_hip_hybrid_destroy(c);
    return rc;
  }
  *out = c;
  return 0;
}

int crabml_hip_hybrid_destroy(crabml_hip_hybrid_t* c) {
  if (!c) return 0;
  (void)hipSetDevice(c->dev->ordinal);
  (void)hipStreamSynchronize(c->dev->stream);
  for (auto& g : c->graphs) {
    if (g.second.second) (void)hipGraphExecDestroy(g.second.second);
    if (g.second.first) (void)hipGraphDestroy(g.second.first);
  }
  for (auto& s : c->seqs)
    if (s.open) pool_free(c->dev, s.slab, s.cap);
  for (auto& a : c->allocs) pool_free(c->dev, a.first, a.second);
  if (c->side) {
    (void)hipStreamSynchronize(c->side);
    (void)hipStreamDestroy(c->side);
  }
  if (c->fork) (void)hipEventDestroy(c->fork);
  if (c->join) (void)hipEventDestroy(c->join);
  if (c->h_seq) (void)hipHostFree(c->h_seq);
  if (c->h_meta) (void)hipHostFree(c->h_meta);
  delete c;
  return 0;
}

int crabml_hip_hybrid_open(crabml_hip_hybrid_t* c, size_t* seq) {
  if (!c || !seq) return CRABML_HIP_BAD_INPUT;
  CH_USE(c->dev);
  size_t i = 0;
  while (i < c->seqs.size() && c->seqs[i].open) i++;
  if (i == c->seqs.size()) c->seqs.emplace_back();
  Seq s;
  CH_TRY(pool_alloc(c->dev, c->slab_bytes, (void**)&s.slab, &s.cap));
  s.open = true;
  c->seqs[i] = s;
  *seq = i;
  return 0;
}

int crabml_hip_hybrid_close(crabml_hip_hybrid_t* c, size_t seq) {
  if (!c) return CRABML_HIP_BAD_INPUT;
  CH_TRY(check_seq(c, seq));
  pool_free(c->dev, c->seqs[seq].slab, c->seqs[seq].cap);  // (one stream: whoever gets it next is ordered behind us)
  c->seqs[seq] = Seq();
  return 0;
}

size_t crabml_hip_hybrid_len(const crabml_hip_hybrid_t* c, size_t seq) { return c && seq < c->seqs.size() ? c->seqs[seq].len : 0; }
size_t crabml_hip_hybrid_slab_bytes(const crabml_hip_hybrid_t* c) { return c ? c->slab_bytes : 0; }

int crabml_hip_hybrid_step(crabml_hip_hybrid_t* c, size_t n, const size_t* seqs, const size_t* counts, const uint32_t* tokens, const size_t* want_counts,
                           const uint32_t* want, float* logits) {
  if (!c || (n && (!seqs || !counts || !tokens))) return CRABML_HIP_BAD_INPUT;
  crabml_hip_device* dev = c->dev;
  CH_LIVE(dev);
  CH_USE(dev);
  CH_FLUSH(dev);
  // everything is checked before anything runs
  bool single = n <= HYB_STEP_ROWS;
  size_t n_tok = 0, n_want = 0;
  std::vector<char> seen(c->seqs.size(), 0);
  for (size_t i = 0; i < n; i++) {
    CH_TRY(check_seq(c, seqs[i]));
    if (seen[seqs[i]]) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: sequence %zu twice in one step", seqs[i]);
    seen[seqs[i]] = 1;
    if (!counts[i]) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: sequence %zu gets no tokens", seqs[i]);
    if (counts[i] > c->cfg.seq_len || c->seqs[seqs[i]].len + counts[i] > c->cfg.seq_len)
      CH_BAIL(dev, CRABML_HIP_TENSOR_ERROR, "hybrid: %zu more tokens do not fit sequence %zu (%zu of %zu used)", counts[i], seqs[i], c->seqs[seqs[i]].len, c->cfg.seq_len);
    for (size_t t = 0; t < counts[i]; t++)
      if (tokens[n_tok + t] >= c->cfg.vocab_size) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: token %u out of range", tokens[n_tok + t]);
    for (size_t k = 0; want_counts && k < want_counts[i]; k++)
      if (!want || want[n_want + k] >= counts[i] || (k && want[n_want + k] <= want[n_want + k - 1]))
        CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: wanted places must ascend inside the new tokens");
    n_tok += counts[i];
    n_want += want_counts ? want_counts[i] : 0;
    single = single && counts[i] == 1;
  }
  if (n_want && !logits) return CRABML_HIP_BAD_INPUT;
  if (n == 0) return 0;
  if (single) {
    CH_TRY(step_begin(c, n, seqs, tokens));
    CH_TRY(run_step(c, (int)n, false));
    for (size_t i = 0; i < n; i++) c->seqs[seqs[i]].len++;
    if (n_want) {
      for (size_t i = 0; i < n; i++)
        if (want_counts[i]) {
          CH_HIP(dev, hipMemcpyAsync(logits, c->st_logits + i * c->vocab, c->vocab * sizeof(float), hipMemcpyDeviceToHost, dev->stream));
          logits += c->vocab;
        }
      CH_HIP(dev, hipStreamSynchronize(dev->stream));
    }
    return 0;
  }
  const size_t cap = c->cfg.pass_rows ? c->cfg.pass_rows : 2048;
  std::vector<Part> parts;
  CH_TRY(pass_alloc(c));
  size_t used = 0, hist = 0, tok = 0, wat = 0;
  for (size_t i = 0; i < n; i++) {
    size_t done = 0, k = 0;
    const size_t nw = want_counts ? want_counts[i] : 0;
    while (done < counts[i]) {
      const size_t back = std::min(c->hist, c->seqs[seqs[i]].len);  // (a part that waits in `parts` is not of this sequence)
      if (used == cap || (hist && hist + back > c->hist_cap)) {
        CH_TRY(run_pass(c, parts, &logits));
        parts.clear();
        used = hist = 0;
        continue;
      }
      Part p;
      p.seq = seqs[i];
      p.n = std::min(counts[i] - done, cap - used);
      p.tokens = tokens + tok + done;
      for (; k < nw && want[wat + k] < done + p.n; k++) p.want.push_back((int)(want[wat + k] - done));
      done += p.n;
      used += p.n;
      hist += back;
      parts.push_back(std::move(p));
    }
    tok += counts[i];
    wat += nw;
  }
  return run_pass(c, parts, &logits);
}

int crabml_hip_hybrid_decode_greedy(crabml_hip_hybrid_t* c, size_t n, const size_t* seqs, const uint32_t* tokens, size_t n_steps, uint32_t* out_tokens) {
  if (!c || !seqs || !tokens || (!out_tokens && n_steps)) return CRABML_HIP_BAD_INPUT;
  crabml_hip_device* dev = c->dev;
  CH_LIVE(dev);
  CH_USE(dev);
  CH_FLUSH(dev);
  if (n == 0 || n > HYB_STEP_ROWS) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: greedy decoding takes 1 to %d sequences, not %zu", HYB_STEP_ROWS, n);
  std::vector<char> seen(c->seqs.size(), 0);
  for (size_t i = 0; i < n; i++) {
    CH_TRY(check_seq(c, seqs[i]));
    if (seen[seqs[i]]) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: sequence %zu twice in one step", seqs[i]);
    seen[seqs[i]] = 1;
    if (tokens[i] >= c->cfg.vocab_size) CH_BAIL(dev, CRABML_HIP_BAD_INPUT, "hybrid: token %u out of range", tokens[i]);
    if (n_steps > c->cfg.seq_len || c->seqs[seqs[i]].len + n_steps > c->cfg.seq_len)
      CH_BAIL(dev, CRABML_HIP_TENSOR_ERROR, "hybrid: %zu steps do not fit sequence %zu (%zu of %zu used)", n_steps, seqs[i], c->seqs[seqs[i]].len, c->cfg.seq_len);
  }
  if (n_steps == 0) return 0;
  CH_TRY(step_begin(c, n, seqs, tokens));
  CH_HIP(dev, hipMemsetAsync(c->st_count, 0, sizeof(int), dev->stream));
  for (size_t s = 0; s < n_steps; s++) CH_TRY(run_step(c, (int)n, true));
  for (size_t i = 0; i < n; i++) c->seqs[seqs[i]].len += n_steps;
  CH_HIP(dev, hipMemcpyAsync(out_tokens, c->st_out, n_steps * n * sizeof(uint32_t), hipMemcpyDeviceToHost, dev->stream));
  CH_HIP(dev, hipStreamSynchronize(dev->stream));
  return 0;
}

}  // extern "C"
