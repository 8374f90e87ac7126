// llmlb-test: native unit tests for the gateway internals (TPS math,
// selection, admission, HTTP parsing, chunked scanner, SSE tap, JSON,
// crypto).  Mirrors the reference's in-file unit-test tier.
// Exit code 0 = all pass.
#include <cstdio>
#include <unistd.h>

#include "http.h"
#include "json.h"
#include "gateway.h"
#include "router.h"
#include "anthropic.h"
#include "db.h"
#include "history.h"
#include "sha256.h"
#include "bpe.h"

using namespace gw;

static int g_failures = 0;
#define CHECK(cond)                                                        \
  do {                                                                     \
    if (!(cond)) {                                                         \
      fprintf(stderr, "FAIL %s:%d: %s\n", __FILE__, __LINE__, #cond);      \
      ++g_failures;                                                        \
    }                                                                      \
  } while (0)

static void test_sha256() {
  // FIPS 180-4 known vectors
  CHECK(sha256_hex("abc") ==
        "ba7816bf8f01cfea414140de5dae2223b00361a396177a9cb410ff61f20015ad");
  CHECK(sha256_hex("") ==
        "e3b0c44298fc1c149afbf4c8996fb92427ae41e4649b934ca495991b7852b855");
  // RFC 4231 HMAC-SHA256 test case 2
  uint8_t mac[32];
  hmac_sha256("Jefe", "what do ya want for nothing?", mac);
  CHECK(hex_encode(mac, 32) ==
        "5bdcc146bf60754e6a042426089575c75a003f089d2739839dec58b964ec3843");
}

static void test_b64() {
  CHECK(b64_encode("hello") == "aGVsbG8=");
  CHECK(b64_decode("aGVsbG8=") == "hello");
  CHECK(b64_encode("a") == "YQ==");
  const std::string bin("\x00\xff\x10""binary", 9);  // embedded NUL
  CHECK(b64_decode(b64_encode(bin, false, true)) == bin);
}

static void test_json() {
  Json v;
  std::string err;
  CHECK(Json::parse(R"({"a":[1,2.5,"x\n",true,null],"b":{"c":-3}})", v,
                    &err));
  CHECK(v["a"].as_arr().size() == 5);
  CHECK(v["a"].as_arr()[1].as_num() == 2.5);
  CHECK(v["a"].as_arr()[2].as_str() == "x\n");
  CHECK(v["b"]["c"].as_int() == -3);
  CHECK(!Json::parse("{", v, &err));
  CHECK(!Json::parse("{\"a\":}", v, &err));
  // unicode escape
  CHECK(Json::parse(R"("é😀")", v));
  CHECK(v.as_str() == "\xc3\xa9\xf0\x9f\x98\x80");
  // round trip
  Json obj = JsonObject{{"x", Json("a\"b")}, {"n", Json(42)}};
  Json back;
  CHECK(Json::parse(obj.dump(), back));
  CHECK(back["x"].as_str() == "a\"b" && back["n"].as_int() == 42);
  // raw field helpers
  CHECK(raw_string_field(R"({"model":"m1","nested":{"model":"no"}})",
                         "model") == "m1");
  CHECK(raw_string_field(R"({"first":"x","model":"m2"})", "model") ==
        "m2");
  CHECK(raw_string_field(R"({"a":{"model":"inner"}})", "model") == "");
}

static void test_http_parse() {
  HttpRequest req;
  std::string raw = "POST /v1/chat/completions?x=1 HTTP/1.1\r\n"
                    "Host: h\r\nContent-Length: 5\r\n\r\nhello";
  CHECK(parse_request_head(raw, req) == 1);
  CHECK(req.method == "POST");
  CHECK(req.path == "/v1/chat/completions");
  CHECK(req.query == "x=1");
  CHECK(req.content_length == 5);
  CHECK(req.keep_alive);
  HttpRequest req2;
  CHECK(parse_request_head("GET / HT", req2) == 0);  // incomplete
  CHECK(parse_request_head("garbage\r\n\r\n", req2) == -1);

  HttpResponse resp;
  std::string rr = "HTTP/1.1 200 OK\r\nTransfer-Encoding: chunked\r\n"
                   "Content-Type: text/event-stream\r\n\r\n";
  CHECK(parse_response_head(rr, resp) == 1);
  CHECK(resp.status == 200 && resp.chunked);
}

static void test_chunked_scanner() {
  // single feed
  ChunkedScanner cs;
  std::string body = "5\r\nhello\r\n3\r\nabc\r\n0\r\n\r\n";
  auto r = cs.scan(body);
  CHECK(r.complete);
  std::string payload;
  for (auto& [off, len] : r.payload) payload += body.substr(off, len);
  CHECK(payload == "helloabc");
  // byte-at-a-time feed (split across TCP segments)
  ChunkedScanner cs2;
  payload.clear();
  bool complete = false;
  for (char c : body) {
    auto rr = cs2.scan(std::string_view(&c, 1));
    for (auto& [off, len] : rr.payload) payload += c;
    if (rr.complete) complete = true;
  }
  CHECK(complete && payload == "helloabc");
  // trailers
  ChunkedScanner cs3;
  std::string wt = "2\r\nhi\r\n0\r\nX-T: v\r\n\r\n";
  auto r3 = cs3.scan(wt);
  CHECK(r3.complete);
}

static void test_sse_tap() {
  SseTap tap;
  tap.feed("data: {\"choices\":[{\"delta\":{\"content\":\"a\"}}]}\n\n");
  tap.feed("data: {\"choices\":[{\"delta\":{\"con");  // split line
  tap.feed("tent\":\"b\"}}]}\n\n");
  tap.feed("data: {\"usage\":{\"prompt_tokens\":7,"
           "\"completion_tokens\":42}}\n\ndata: [DONE]\n\n");
  CHECK(tap.completion_tokens() == 42);
  CHECK(tap.prompt_tokens() == 7);
  CHECK(tap.saw_done());
  // fallback estimate without usage
  SseTap tap2;
  for (int i = 0; i < 5; ++i)
    tap2.feed("data: {\"choices\":[{\"delta\":{\"content\":\"x\"}}]}\n\n");
  CHECK(tap2.completion_tokens() == 5);
  // Responses-API usage field names
  SseTap tap3;
  tap3.feed("data: {\"type\":\"response.completed\",\"response\":{"
            "\"usage\":{\"input_tokens\":3,\"output_tokens\":9}}}\n\n");
  CHECK(tap3.completion_tokens() == 9 && tap3.prompt_tokens() == 3);
}

static void test_tps_and_selection() {
  // EMA alpha 0.2 (balancer/types.rs:102-118)
  TpsState st;
  st.update(100, 1.0, 0.2, 1000);
  CHECK(st.score(1000) == 100.0);
  st.update(200, 1.0, 0.2, 2000);
  CHECK(st.score(2000) > 119.9 && st.score(2000) < 120.1);
  CHECK(st.score(2000 + 121000) == 0.0);  // stale after 120 s
  st.reset();
  CHECK(st.score(2000) == 0.0);

  // selection: TPS-desc with RR tie-break + admission
  auto mk = [](const char* id) {
    auto ep = std::make_shared<Endpoint>();
    ep->id = id;
    ep->status = EndpointStatus::kOnline;
    return ep;
  };
  RouteTable table;
  ModelRoute route;
  route.model_key = "m";
  route.canonical = "m";
  route.rr = std::make_shared<std::atomic<uint64_t>>(0);
  for (const char* id : {"e1", "e2", "e3"}) {
    route.endpoints.push_back(mk(id));
    route.upstream_ids.push_back("m");
    route.tps.push_back(std::make_shared<TpsState>());
    route.caps |= kCapChat;
  }
  table.by_model["m"] = route;
  AdmissionConfig adm;
  // all scores 0 -> pure round robin over all three
  std::string seen;
  for (int i = 0; i < 6; ++i)
    seen += select_endpoint(table, "m", ApiKind::kChat, adm, 5000).ep->id;
  CHECK(seen.find("e1") != std::string::npos &&
        seen.find("e2") != std::string::npos &&
        seen.find("e3") != std::string::npos);
  // e2 earns the best TPS -> always selected
  route.tps[1]->update(500, 1.0, 0.2, 5000);
  table.by_model["m"] = route;
  for (int i = 0; i < 4; ++i)
    CHECK(select_endpoint(table, "m", ApiKind::kChat, adm, 5000).ep->id ==
          "e2");
  // admission: e2 beyond the 80% reject threshold -> next best
  route.endpoints[1]->active = 90;  // of max 100
  CHECK(select_endpoint(table, "m", ApiKind::kChat, adm, 5000).ep->id !=
        "e2");
  // delayed-admission arm (balancer/mod.rs:2255-2270): picked endpoint
  // between 50% and 80% load -> 10..100 ms hold; below 50% -> none
  route.endpoints[1]->active = 0;
  route.endpoints[0]->active = 65;   // 65% -> delay = 10 + 0.5*90 = 55
  route.tps[0]->update(900, 1.0, 0.2, 5000);  // make e1 win selection
  route.tps[1]->reset();
  table.by_model["m"] = route;
  {
    auto r2 = select_endpoint(table, "m", ApiKind::kChat, adm, 5000);
    CHECK(r2.ep->id == "e1");
    CHECK(r2.delay_ms >= 50 && r2.delay_ms <= 60);
    route.endpoints[0]->active = 10;  // 10% -> no delay
    auto r3 = select_endpoint(table, "m", ApiKind::kChat, adm, 5000);
    CHECK(r3.delay_ms == 0);
    route.endpoints[0]->active = 0;
    route.tps[0]->reset();
  }
  route.endpoints[1]->active = 90;   // restore state for HBM-gate test
  // HBM gate: e1+e3 over budget and e2 busy -> 429
  for (auto& ep : route.endpoints) {
    std::lock_guard<std::mutex> lk(ep->gpu_mu);
    ep->gpu.hbm_total_gb = 288;
    ep->gpu.hbm_used_gb = 280;  // 97% > 92% budget
    ep->gpu.updated_ms = 5000;
  }
  auto res = select_endpoint(table, "m", ApiKind::kChat, adm, 5000);
  CHECK(res.err_status == 429);
  // unknown model -> 404
  CHECK(select_endpoint(table, "nope", ApiKind::kChat, adm, 5000)
            .err_status == 404);
  // offline endpoints -> 503
  for (auto& ep : route.endpoints) ep->status = EndpointStatus::kOffline;
  table.by_model["m"] = route;
  CHECK(select_endpoint(table, "m", ApiKind::kChat, adm, 5000)
            .err_status == 503);
}

static void test_lease() {
  auto ep = std::make_shared<Endpoint>();
  ep->status = EndpointStatus::kOnline;
  {
    RequestLease lease(ep, nullptr, "m", ApiKind::kChat);
    CHECK(ep->active.load() == 1);
    lease.complete_success(10);
    CHECK(ep->active.load() == 0);
    CHECK(ep->consecutive_failures.load() == 0);
  }
  CHECK(ep->total_failures.load() == 0);
  {
    RequestLease lease(ep, nullptr, "m", ApiKind::kChat);
    // dropped without completion -> counted as failure (lease.rs:71)
  }
  CHECK(ep->active.load() == 0);
  CHECK(ep->total_failures.load() == 1);
  // move semantics: only the final owner releases
  {
    RequestLease a(ep, nullptr, "m", ApiKind::kChat);
    RequestLease b = std::move(a);
    CHECK(ep->active.load() == 1);
    b.complete_success(1);
  }
  CHECK(ep->active.load() == 0);
}

static void test_audit_archive() {
  // archive old audit rows to a second DB; live chain re-anchors
  std::string base = "/tmp/llmlb_ut_audit.sqlite3";
  std::string arch = base + ".audit-archive.sqlite3";
  remove(base.c_str());
  remove(arch.c_str());
  {
    Db db;
    std::string err;
    CHECK(db.open(base, &err));
    CHECK(db.migrate(&err));
    HistoryWriter hw(&db, 7);
    hw.start();  // archive configured after the loop's first cleanup
                 // pass so the explicit call below does the move
    int64_t now = wall_ms();
    for (int i = 0; i < 10; ++i) {
      AuditRecord a;
      a.ts_ms = now - (int64_t)(10 - i) * 86400 * 1000 * 20;  // 200..20d old
      a.method = "GET";
      a.path = "/x";
      a.status = 200;
      a.duration_ms = 1.0;
      hw.audit(std::move(a));
    }
    for (int spin = 0; spin < 100; ++spin) {
      std::vector<DbRow> rows;
      db.exec("SELECT COUNT(*) FROM audit_log", {}, &rows);
      if (!rows.empty() && rows[0][0].i == 10) break;
      usleep(20000);
    }
    std::string err2;
    CHECK(hw.verify_audit_chain(&err2));
    hw.set_audit_archive(arch, 90);
    // archive everything older than 90 days (first 6 records)
    int moved = hw.archive_audit_now(now - 90LL * 86400 * 1000, &err2);
    CHECK(moved == 6);
    std::vector<DbRow> rows;
    db.exec("SELECT COUNT(*) FROM audit_log", {}, &rows);
    CHECK(rows[0][0].i == 4);
    // live chain still verifies via the anchored tip
    CHECK(hw.verify_audit_chain(&err2));
    // idempotent: nothing else old
    CHECK(hw.archive_audit_now(now - 90LL * 86400 * 1000, &err2) == 0);
    hw.stop();
  }
  {
    // the archive file holds the moved rows and chains from genesis
    Db adb;
    std::string err;
    CHECK(adb.open(arch, &err));
    std::vector<DbRow> rows;
    CHECK(adb.exec("SELECT prev_hash,hash FROM audit_log ORDER BY id", {},
                   &rows));
    CHECK(rows.size() == 6);
    if (rows.size() == 6)
      CHECK(rows[0][0].str() == sha256_hex("genesis"));
  }
  remove(base.c_str());
  remove(arch.c_str());
}

static void test_anthropic_stream_encoder_fragmented() {
  // OpenAI SSE -> Anthropic SSE re-encode must produce the same event
  // sequence whether fed whole or byte-at-a-time
  const std::string in =
      "data: {\"choices\":[{\"delta\":{\"role\":\"assistant\"}}]}\n\n"
      "data: {\"choices\":[{\"delta\":{\"content\":\"Hel\"}}]}\n\n"
      "data: {\"choices\":[{\"delta\":{\"content\":\"lo\"}}]}\n\n"
      "data: {\"choices\":[{\"delta\":{},\"finish_reason\":\"stop\"}]"
      ",\"usage\":{\"prompt_tokens\":3,\"completion_tokens\":2}}\n\n"
      "data: [DONE]\n\n";
  std::string whole, frag;
  {
    AnthropicStreamEncoder enc("m");
    enc.feed(in, whole);
    enc.finish(whole);
  }
  {
    AnthropicStreamEncoder enc("m");
    for (char ch : in) enc.feed(std::string_view(&ch, 1), frag);
    enc.finish(frag);
  }
  // normalise the per-message random id before comparing
  auto strip_id = [](std::string s) {
    size_t p = 0;
    while ((p = s.find("msg_", p)) != std::string::npos) {
      s.replace(p, 4 + 36, "msg_X");
      p += 5;
    }
    return s;
  };
  CHECK(strip_id(whole) == strip_id(frag));
  CHECK(whole.find("message_start") != std::string::npos);
  CHECK(whole.find("content_block_delta") != std::string::npos);
  CHECK(whole.find("Hel") != std::string::npos);
  CHECK(whole.find("message_stop") != std::string::npos);
  CHECK(whole.find("end_turn") != std::string::npos);
}

static void test_permission_matrix() {
  // exact token matching: no substring grants
  CHECK(!AuthStore::perms_grant("badminton", "admin"));
  CHECK(!AuthStore::perms_grant("inference-disabled", "openai.inference"));
  CHECK(!AuthStore::perms_grant("inferenc", "openai.inference"));
  CHECK(AuthStore::perms_grant("admin", "users.manage"));
  CHECK(AuthStore::perms_grant("a,admin,b", "logs.read"));
  // legacy "inference" covers the two openai scopes only
  CHECK(AuthStore::perms_grant("inference", "openai.inference"));
  CHECK(AuthStore::perms_grant("inference", "openai.models.read"));
  CHECK(!AuthStore::perms_grant("inference", "endpoints.manage"));
  // scoped keys: exact scope + no cross-grant (the 11-scope matrix)
  const char* scopes[] = {"openai.inference",  "openai.models.read",
                          "endpoints.read",    "endpoints.manage",
                          "api_keys.manage",   "users.manage",
                          "invitations.manage","models.manage",
                          "registry.read",     "logs.read",
                          "metrics.read"};
  for (const char* a : scopes)
    for (const char* b : scopes)
      CHECK(AuthStore::perms_grant(a, b) == (strcmp(a, b) == 0));
  // whitespace + multi-token lists
  CHECK(AuthStore::perms_grant(" endpoints.read , metrics.read ",
                               "metrics.read"));
  CHECK(!AuthStore::perms_grant("", "openai.inference"));
  // loopback helper
  CHECK(is_loopback_ip("127.0.0.1"));
  CHECK(is_loopback_ip("::1"));
  CHECK(is_loopback_ip("::ffff:127.0.0.1"));
  CHECK(!is_loopback_ip("10.0.0.5"));
  CHECK(!is_loopback_ip("1270.0.0.1"));
}

static void test_secure_random() {
  unsigned char a[32] = {0}, b[32] = {0};
  CHECK(secure_random_bytes(a, sizeof a));
  CHECK(secure_random_bytes(b, sizeof b));
  CHECK(memcmp(a, b, sizeof a) != 0);  // astronomically unlikely equal
}


static void test_bpe_counts() {
  BpeTokenizer bpe;
  CHECK(bpe.load("data/llmlb.tiktoken") ||
        bpe.load("gateway/data/llmlb.tiktoken"));
  // golden counts computed by the HF tokenizer that trained the table
  // (gateway/data/bpe_golden.json) — verifies pre-split + merge parity
  CHECK(bpe.count("Hello, world!") == 4);
  CHECK(bpe.count("The quick brown fox jumps over the lazy dog.") == 13);
  CHECK(bpe.count("def fibonacci(n):\n    return n if n < 2 else fibonacci(n-1) + fibonacci(n-2)\n") == 40);
  CHECK(bpe.count("Streaming tokens per second is the headline metric for LLM serving gateways.") == 20);
  CHECK(bpe.count("   indented\ttext with   runs of whitespace\n\n") == 11);
  CHECK(bpe.count("numbers 12345 and 2026-09-14 09:30:00") == 17);
  CHECK(bpe.count("don't can't we'll they're I'm you've he'd") == 14);
  CHECK(bpe.count("") == 0);
  CHECK(bpe.count("a") == 1);
  CHECK(BpeTokenizer::heuristic_count("abcdefgh") == 2);
}

static void test_caps_csv() {
  CHECK(caps_from_csv("chat,embeddings") == (kCapChat | kCapEmbeddings));
  CHECK(caps_to_csv(kCapAudioSpeech) == "audio_speech");
  CHECK(caps_from_csv(caps_to_csv(kCapChat | kCapImageGen)) ==
        (kCapChat | kCapImageGen));
}

int main() {
  test_sha256();
  test_b64();
  test_json();
  test_http_parse();
  test_chunked_scanner();
  test_sse_tap();
  test_tps_and_selection();
  test_lease();
  test_audit_archive();
  test_anthropic_stream_encoder_fragmented();
  test_permission_matrix();
  test_bpe_counts();
  test_secure_random();
  test_caps_csv();
  if (g_failures == 0) {
    printf("llmlb-test: all native unit tests passed\n");
    return 0;
  }
  fprintf(stderr, "llmlb-test: %d failure(s)\n", g_failures);
  return 1;
}
